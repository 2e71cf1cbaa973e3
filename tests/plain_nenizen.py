"""A plain, slow Nenizen: whole sequences, float64, no cache, one function per mechanism.

It shares nothing with the engine: it computes every token of a sequence from scratch, makes every head's keys and
values in full, and walks the layers of a loop as often as they run.  The tests compare the engine with it.
"""

from __future__ import annotations

import numpy as np

from plain_mafosun import read_config, read_weights  # noqa: F401  (reading the two files of a model folder)


# ------------------------------------------------------------------------------ mechanisms
def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate(x, positions, base, interleaved):
    """x [T, ..., d], all d values turned: pair i by the angle p * base^(-2i/d); the pairs are (2i, 2i + 1) or
    (i, i + d/2)."""
    d = x.shape[-1]
    if d == 0:
        return x
    i = np.arange(d // 2)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * base ** (-2.0 * i / d)
    angle = angle.reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (d // 2,))
    c, s = np.cos(angle), np.sin(angle)
    first, second = (2 * i, 2 * i + 1) if interleaved else (i, i + d // 2)
    out = np.empty_like(x)
    out[..., first] = x[..., first] * c - x[..., second] * s
    out[..., second] = x[..., second] * c + x[..., first] * s
    return out


def visible(t, window=None):
    """[T, T] of booleans: query i sees key j (the latest ``window`` positions, itself included, or all before it)."""
    i, j = np.arange(t)[:, None], np.arange(t)[None, :]
    return (j <= i) if window is None else (j <= i) & (i - j < window)


def softmax_mix(scores, mask, v, sink=None):
    """scores [H, T, T], v [T, H, e] -> [T, H, e]; ``sink`` [H]: exp(sink) joins every denominator of its head."""
    s = np.where(mask[None], scores, -np.inf)
    m = s.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink[:, None, None])
    e = np.exp(s - m)
    den = e.sum(-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink[:, None, None] - m)
    return np.einsum("hij,jhe->ihe", e / den, v)


def latent_keys(h, positions, w, p, m, eps, interleaved):
    """The latent [T, kv_rank] after its norm and the turned key part [T, rot_dim] that all heads share."""
    row = h @ w[p + "dkv"].T
    rank = m["kv_rank"]
    return rms_norm(row[:, :rank], w[p + "dkv.norm"], eps), rotate(row[:, rank:], positions, m["rot"]["base"], interleaved)


def clipped_gate(g, u, limit):
    """min(g, limit) sigmoid(1.702 min(g, limit)) (clamp(u, -limit, limit) + 1)"""
    g = np.minimum(g, limit)
    return g * sigmoid(1.702 * g) * (np.clip(u, -limit, limit) + 1.0)


def route(z, top, margins=None):
    """Softmax scores of z [T, E]; the ``top`` largest of every token and those scores as weights.  ``margins`` (a list)
    receives, per token, the distance between the last expert chosen and the first one not as a part of the logits'
    spread (infinite where all are chosen)."""
    s = np.exp(z - z.max(-1, keepdims=True))
    s /= s.sum(-1, keepdims=True)
    ids = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    if margins is not None:
        ordered = -np.sort(-z, axis=-1)
        gap = ordered[:, top - 1] - ordered[:, top] if top < z.shape[1] else np.full(z.shape[0], np.inf)
        margins.append(gap / np.maximum(ordered[:, 0] - ordered[:, -1], 1e-30))
    return ids, np.take_along_axis(s, ids, axis=-1)


def gated_ff(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def enter_pass(x, x0, w, number):
    """What stands before the first layer of a pass of the loop."""
    return np.concatenate([x, x0], axis=-1) @ w["loop.in"].T + w["loop.step"][number]


# ---------------------------------------------------------------------------------- layers
KINDS = {  # queries through a latent, neighbouring pairs, a window, a sink a head, the gate
    "latent_attention": dict(latent_q=False, interleaved=True, window=False, sink=False, gate="values"),
    "latent_attention_2": dict(latent_q=True, interleaved=False, window=True, sink=False, gate="heads"),
    "latent_attention_3": dict(latent_q=True, interleaved=False, window=False, sink=True, gate=None),
}


def mixer(kind, h, positions, w, p, m, eps):
    k = KINDS[kind]
    t, heads, dim, rot, e = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T if k["latent_q"] else h @ w[p + "q"].T
    q = q.reshape(t, heads, dim + rot)
    q_turned = rotate(q[..., dim:], positions, m["rot"]["base"], k["interleaved"])
    c, k_turned = latent_keys(h, positions, w, p, m, eps, k["interleaved"])
    keys = (c @ w[p + "uk"].T).reshape(t, heads, dim)
    values = (c @ w[p + "uv"].T).reshape(t, heads, e)
    scores = (np.einsum("ihd,jhd->hij", q[..., :dim], keys) + np.einsum("ihd,jd->hij", q_turned, k_turned)) * m["scale"]
    o = softmax_mix(scores, visible(t, m["mask"]["size"] if k["window"] else None), values, w[p + "sink"] if k["sink"] else None)
    if k["gate"] == "heads":
        o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    o = o.reshape(t, heads * e)
    if k["gate"] == "values":
        o = o * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def feed_forward(h, w, p, mlp, margins=None):
    if mlp["kind"] == "dense":
        return clipped_gate(h @ w[p + "gate"].T, h @ w[p + "up"].T, mlp["limit"]) @ w[p + "down"].T
    ids, weights = route(h @ w[p + "router"].T, mlp["router"]["top"], margins)
    out = np.zeros_like(h) if mlp.get("shared") is None else gated_ff(h, w, p + "shared.")
    for e in range(mlp["router"]["experts"]):
        rows, place = np.nonzero(ids == e)
        if len(rows):
            out[rows] += weights[rows, place][:, None] * gated_ff(h[rows], w, f"{p}e{e}.")
    return out


def runs(cfg):
    """(layer, number of the pass whose entrance comes before it or None) in the order in which layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, w: dict, tokens, streams=None, margins=None):
    """Logits [T, vocab] of the whole sequence; ``streams`` (a list) receives the stream after every layer that runs,
    ``margins`` one array [T] for every run of a layer of routed experts."""
    eps = cfg["norm"]["eps"]
    positions = np.arange(len(tokens))
    x = x0 = w["embed"][np.asarray(tokens, dtype=np.int64)] * cfg["embedding"]["scale"]
    for i, entrance in runs(cfg):
        p, layer = f"l{i}.", cfg["layers"][i]
        if entrance is not None:
            x = enter_pass(x, x0, w, entrance)
        y = mixer(layer["type"], rms_norm(x, w[p + "norm1"], eps), positions, w, p + "mix.", layer["mixer"], eps)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"], margins)
            x = x + rms_norm(y, w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.copy())
    logits = rms_norm(x, w["final.norm"], eps) @ w["embed"].T
    cap = cfg.get("logit_softcap")
    return logits if not cap else cap * np.tanh(logits / cap)


def load(folder):
    return read_config(folder), read_weights(folder)
