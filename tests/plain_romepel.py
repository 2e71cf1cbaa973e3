"""Plain, slow implementation of the Romepel decoder: whole sequences, no cache, one function
for each mechanism, float64 on the CPU.

It shares no code with the engine: config.json is read with ``json``, the weights with the
``safetensors`` package.  Notation: ``x`` [T, W] is the residual stream of one sequence whose
positions are 0..T-1, ``h`` a sublayer's input, weights are stored [out, in].
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F = torch.float64


def read_config(model_dir) -> dict:
    return json.loads((Path(model_dir) / "config.json").read_text())


def read_weights(model_dir) -> dict:
    from safetensors import safe_open

    out = {}
    with safe_open(str(Path(model_dir) / "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            t = f.get_tensor(name)
            out[name] = t if t.dtype in (torch.int32, torch.int64) else t.to(F)
    return out


# ------------------------------------------------------------------------------------------
# small pieces
# ------------------------------------------------------------------------------------------
def unit_rms(x, eps: float):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_plain_weight(x, w, eps: float):
    return unit_rms(x, eps) * w


def norm_zero_centred(x, w, eps: float):
    """The stored tensor is the factor less one."""
    return unit_rms(x, eps) * (1.0 + w)


def positioned_embedding(ids, table, position_table, first: int = 0):
    """Row of the token plus row of its position; the sequence starts at position ``first``."""
    ids = torch.as_tensor(ids, dtype=torch.int64)
    return table[ids] + position_table[first:first + ids.shape[0]]


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def xielu(z, act):
    """``act`` = (p, q).  Above zero a parabola with coefficient softplus(p), below it exp(z) - 1 - z with coefficient
    1/2 + softplus(q); half of z is added on both sides."""
    up, down = softplus(act[0]), 0.5 + softplus(act[1])
    neg = torch.clamp(z, max=0.0)
    return torch.where(z > 0, up * z * z, down * (torch.expm1(neg) - neg)) + 0.5 * z


def dense_feed_forward(h, up, up_b, act, down, down_b):
    return xielu(h @ up.t() + up_b, act) @ down.t() + down_b


def distance_slopes(heads: int):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=F)


def query_temperature(positions, coef: float, every: float):
    """1 + coef * ln(floor((p + 1) / every) + 1) at every position p."""
    p = torch.as_tensor(positions, dtype=F)
    return 1.0 + coef * torch.log(torch.floor((p + 1.0) / every) + 1.0)


def window_mask(queries, keys, window):
    """[len(queries), len(keys)]: which keys a query sees (itself and the window - 1 positions before it)."""
    d = torch.as_tensor(queries).reshape(-1, 1) - torch.as_tensor(keys).reshape(1, -1)
    return (d >= 0) & (d < window) if window else d >= 0


def softmax(s):
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def biased_attention(q, k, v, first: int, scale: float, window, slopes, temperature):
    """q [n, H, dim] of the positions first .. first + n, k [S, G, dim] and v [S, G, vdim] of the positions 0 .. S;
    ``temperature`` [n] multiplies the queries; returns [n, H, vdim]."""
    n, heads, groups = q.shape[0], q.shape[1], k.shape[1]
    pos = torch.arange(first, first + n)
    keys = torch.arange(k.shape[0])
    visible = window_mask(pos, keys, window)
    distance = (pos.reshape(-1, 1) - keys.reshape(1, -1)).to(F)
    out = []
    for h in range(heads):
        g = h // (heads // groups)
        s = ((q[:, h] * temperature.reshape(-1, 1)) @ k[:, g].t()) * scale - slopes[h] * distance
        out.append(softmax(s.masked_fill(~visible, float("-inf"))) @ v[:, g])
    return torch.stack(out, dim=1)


# ------------------------------------------------------------------------------------------
# mixers
# ------------------------------------------------------------------------------------------
def attention(h, w, p: str, m: dict):
    t = h.shape[0]
    nh, nkv, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].t() + w[p + "q.b"]).reshape(t, nh, dim)
    k = (h @ w[p + "k"].t() + w[p + "k.b"]).reshape(t, nkv, dim)
    v = (h @ w[p + "v"].t() + w[p + "v.b"]).reshape(t, nkv, vd)
    temp = m.get("q_temp")
    factor = query_temperature(range(t), temp["coef"], temp["every"]) if temp else torch.ones(t, dtype=F)
    window = m["mask"]["size"] if m.get("mask") else None
    o = biased_attention(q, k, v, 0, m["scale"], window, distance_slopes(nh), factor)
    return o.reshape(t, nh * vd) @ w[p + "o"].t()


def gla_walk(q, k, v, alpha):
    """S <- diag(alpha_t) S + k_t v_t^T from zero, o_t = S^T q_t; q, k, alpha [T, H, dim], v [T, H, vdim]."""
    state = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=F)
    out = []
    for i in range(q.shape[0]):
        state = alpha[i].unsqueeze(-1) * state + k[i].unsqueeze(-1) * v[i].unsqueeze(-2)
        out.append((state * q[i].unsqueeze(-1)).sum(dim=1))
    return torch.stack(out)


def gla(h, w, p: str, m: dict, eps: float):
    t = h.shape[0]
    nh, dim, vd = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].t()).reshape(t, nh, dim) * dim ** -0.5
    k = (h @ w[p + "k"].t()).reshape(t, nh, dim)
    v = (h @ w[p + "v"].t()).reshape(t, nh, vd)
    z = (h @ w[p + "a1"].t()) @ w[p + "a2"].t() + w[p + "a2.b"]
    alpha = torch.pow(torch.sigmoid(z), 1.0 / m["tau"]).reshape(t, nh, dim)
    o = norm_plain_weight(gla_walk(q, k, v, alpha), w[p + "norm"], eps).reshape(t, nh * vd)
    g = h @ w[p + "g"].t()
    return (o * (g * torch.sigmoid(g))) @ w[p + "o"].t()


# ------------------------------------------------------------------------------------------
# the model
# ------------------------------------------------------------------------------------------
def forward(cfg: dict, w: dict, ids, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = positioned_embedding(ids, w["embed"], w["pos"])
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = norm_zero_centred(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = attention(h, w, p + "mix.", m)
        elif layer["type"] == "gla":
            y = gla(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + norm_zero_centred(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            h = norm_zero_centred(x, w[p + "norm2"], eps)
            q = p + "mlp."
            y = dense_feed_forward(h, w[q + "up"], w[q + "up.b"], w[q + "act"], w[q + "down"], w[q + "down.b"])
            x = x + norm_zero_centred(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    logits = norm_zero_centred(x, w["final.norm"], eps) @ w["head"].t()
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
