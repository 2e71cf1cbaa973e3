"""Nenizen on the GPU against the plain implementation (plain_nenizen.py): every mechanism alone, then whole models of
small configurations through the step function, the scheduler and the replay program.

The weights are drawn here with a spread that keeps activations of order one and scores peaked.  For keys that must or
must not be seen, a pair of tokens is made loud: one query's score with one key stands out among hundreds."""

import copy
import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
import plain_nenizen as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def ops():
    from from_scratch_inference_engine_amd import ops as o

    o.load()
    return o


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale


def rel(got, ref):
    got, ref = np.asarray(got, dtype=np.float64), np.asarray(ref, dtype=np.float64)
    return float(np.abs(got - ref).max() / max(np.abs(ref).max(), 1e-30))


def tol(dtype, f32=2e-5, bf16=2.0 ** -6):
    return f32 if dtype == torch.float32 else bf16


def f64(t):
    return t.double().cpu().numpy()


# ------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("limit, slope", [(0.8, 1.702), (3.0, 0.5), (100.0, 2.5)])
def test_clipped_gates_alone(ops, dtype, limit, slope):
    """Gates and up values around both limits and far beyond them, a gate far below zero (which nothing cuts off)."""
    x = rnd((7, 2 * 90), 1, 2.0)
    x[0, :12] = torch.tensor([limit, limit, limit + 50, -limit - 50, -limit, -limit, -60.0, limit, 0.0, 5.0, -0.0, -limit])
    x = x.to(dtype)
    ref = clipped_reference(f64(x)[:, 0::2], f64(x)[:, 1::2], limit, slope)
    act = ops.GateAct("clipped", limit=limit, slope=slope)
    got = ops.swiglu(x.cuda(), act=act)
    assert rel(f64(got), ref) <= tol(dtype, 2e-6, 2.0 ** -8)
    odd = ops.swiglu(x[:, :2 * 33].contiguous().cuda(), act=act)  # (a width that is no multiple of four)
    assert rel(f64(odd), ref[:, :33]) <= tol(dtype, 2e-6, 2.0 ** -8)


def clipped_reference(g, u, limit, slope):
    g = np.minimum(g, limit)
    return g / (1.0 + np.exp(-slope * g)) * (np.clip(u, -limit, limit) + 1.0)


@pytest.mark.parametrize("m, k, inter", [(1, 64, 20), (5, 256, 66), (16, 128, 130), (33, 256, 64), (64, 384, 512), (100, 256, 1024)])
def test_clipped_gates_in_the_products(ops, m, k, inter):
    """In the epilogue of the few-rows product, of the one that shares x through LDS (from rows and from the
    fragment-ordered copy) and behind a product of its own."""
    limit, slope = 0.9, 1.702
    x = rnd((m, k), 1, 1.5).bfloat16()
    w = rnd((2 * inter, k), 2, k ** -0.5).bfloat16()  # gate and up rows in turn
    both = f64(x) @ f64(w).T
    ref = clipped_reference(both[:, 0::2], both[:, 1::2], limit, slope)
    act = ops.GateAct("clipped", limit=limit, slope=slope)
    x, w = x.cuda(), w.cuda()
    if m <= 16:
        assert rel(f64(ops.gemm_mfma_skinny_gated(x, w, act)), ref) <= 2.0 ** -7
        plain_silu = both[:, 0::2] * plain.sigmoid(both[:, 0::2]) * both[:, 1::2]
        assert rel(f64(ops.gemm_mfma_skinny_gated(x, w, "silu")), plain_silu) <= 2.0 ** -7
    if k % 128 == 0 and inter % 2 == 0 and m <= 64:
        assert rel(f64(ops.gemm_mfma_wide_swiglu(x, w, act=act)), ref) <= 2.0 ** -7
    if k % 128 == 0 and inter % 2 == 0 and ops.gemm_mfma_wide_takes(m, ops.fragment_order(w), 1, True):
        assert rel(f64(ops.gemm_mfma_wide_swiglu(x, ops.fragment_order(w), act=act)), ref) <= 2.0 ** -7


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 6, 40, 90])
def test_dense_feed_forward_with_a_clipped_gate(ops, dtype, rows):
    from from_scratch_inference_engine_amd.parts import SwiGLU

    h, ff, limit = 136, 72, 1.1
    part = SwiGLU(h, ff, ops.GateAct("clipped", limit=limit, slope=1.702))
    w = {n: rnd(s, i, 1.5 * s[1] ** -0.5).to(dtype) for i, (n, s) in enumerate((("gate", (ff, h)), ("up", (ff, h)), ("down", (h, ff))))}
    part.gate_up_weight = torch.stack([w["gate"], w["up"]], 1).reshape(2 * ff, h).contiguous().cuda()
    part.down_weight = w["down"].cuda()
    x = rnd((rows, h), 9).to(dtype)
    got = part.forward(x.cuda(), SimpleNamespace(partial_sums_ok=False))
    ref = plain.feed_forward(f64(x), {n: f64(t) for n, t in w.items()}, "", {"kind": "dense", "limit": limit})
    assert rel(f64(got), ref) <= tol(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("t, hidden, ff, experts, top, shared_ff", [(9, 64, 32, 6, 2, 48), (70, 90, 34, 5, 5, 18), (300, 40, 18, 4, 1, None),
                                                                   (1, 128, 64, 16, 3, 128), (24, 256, 40, 3, 2, 520)])
def test_routed_experts_beside_a_shared_one(ops, dtype, t, hidden, ff, experts, top, shared_ff):
    """The chosen experts' softmax scores are not renormalised; the shared expert's output joins the sum whole, rounded or
    as partial sums."""
    from from_scratch_inference_engine_amd.parts import RoutedExperts, SwiGLU

    names = {"router": (experts, hidden)}
    for e in range(experts):
        names.update({f"e{e}.gate": (ff, hidden), f"e{e}.up": (ff, hidden), f"e{e}.down": (hidden, ff)})
    if shared_ff:
        names.update({"shared.gate": (shared_ff, hidden), "shared.up": (shared_ff, hidden), "shared.down": (hidden, shared_ff)})
    w = {n: rnd(s, 100 + i, (10.0 if n == "router" else 1.5) * s[1] ** -0.5).to(dtype) for i, (n, s) in enumerate(names.items())}

    def gated(p, width):
        part = SwiGLU(hidden, width)
        part.gate_up_weight = torch.stack([w[p + "gate"], w[p + "up"]], 1).reshape(2 * width, hidden).contiguous().cuda()
        part.down_weight = w[p + "down"].cuda()
        return part
    part = RoutedExperts(hidden, ff, experts, top, scores="softmax", renorm=False, correction=False, gated="silu",
                         shared=gated("shared.", shared_ff) if shared_ff else None)
    part.router_weight = w["router"].cuda()
    part.up_weight = torch.cat([torch.stack([w[f"e{e}.gate"], w[f"e{e}.up"]], 1).reshape(2 * ff, hidden) for e in range(experts)]).contiguous().cuda()
    part.down_weight = torch.cat([w[f"e{e}.down"] for e in range(experts)]).contiguous().cuda()
    x = rnd((t, hidden), 3).to(dtype)
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top}, "shared": {"ff": shared_ff} if shared_ff else None}
    ref = plain.feed_forward(f64(x), {n: f64(v) for n, v in w.items()}, "", mlp)
    for sums in (False, True):
        got = part.forward(x.cuda(), SimpleNamespace(partial_sums_ok=sums))
        assert got.dtype == torch.float32 and rel(f64(got), ref) <= tol(dtype)


def test_sum_of_experts_takes_a_shared_output_in_every_form(ops):
    t, top, h = 11, 2, 52
    rows, slot_of = rnd((t * top, h), 1), torch.randperm(t * top, generator=torch.Generator().manual_seed(2)).int()
    base = f64(rows)[slot_of.long().numpy()].reshape(t, top, h).sum(1)
    for width in (52, 51):
        cut = rows[:, :width].contiguous()
        parts = rnd((3, t, width), 4)
        for shared in (None, parts[0].contiguous(), parts[0].bfloat16().contiguous(), parts, parts[:1].contiguous()):
            extra = 0.0 if shared is None else f64(shared) if shared.ndim == 2 else f64(shared).sum(0)
            got = ops.moe_combine(cut.cuda(), slot_of.cuda(), t, top, shared=None if shared is None else shared.cuda())
            assert rel(f64(got), base[:, :width] + extra) <= 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [64, 90, 257, 2304, 4104])
def test_the_stream_goes_out_and_starts_again(ops, dtype, hidden):
    """Nothing pending, a delta as it is or through its norm, rounded, float32 or in partial sums: out receives the stream
    in columns of wider rows (whose others stay), every row of the stream becomes the given vector."""
    eps = 1e-3
    for t in (5, 150):
        res, w, start = rnd((t, hidden), 1, 3.0), rnd((hidden,), 2) + 1.0, rnd((hidden,), 5)
        for kind in ("none", "same", "f32", "parts"):
            delta = {"none": None, "same": rnd((t, hidden), 3).to(dtype), "f32": rnd((t, hidden), 3), "parts": rnd((4, t, hidden), 3)}[kind]
            whole = 0.0 if delta is None else f64(delta) if delta.ndim == 2 else f64(delta).sum(0)
            for post in ((False,) if delta is None else (False, True)):
                ref = f64(res) + (plain.rms_norm(whole, f64(w), eps) if post else whole)
                r = res.clone().cuda()
                rows = torch.full((t, 2 * hidden + 8), 7.0, dtype=dtype).cuda()
                ops.stream_out(r, None if delta is None else delta.cuda(), w.cuda() if post else None, eps, rows[:, 4:4 + hidden], start.cuda())
                assert rel(f64(rows[:, 4:4 + hidden]), ref) <= tol(dtype, 2e-6, 2.0 ** -8), (kind, post)
                assert torch.equal(r.cpu(), start.expand(t, hidden)), (kind, post)
                assert (rows[:, :4] == 7.0).all() and (rows[:, 4 + hidden:] == 7.0).all()
        rows = torch.full((t, hidden + 3), 7.0, dtype=dtype).cuda()
        ops.round_columns(res.cuda(), rows[:, 2:2 + hidden])
        assert torch.equal(rows[:, 2:2 + hidden].cpu(), res.to(dtype)) and (rows[:, :2] == 7.0).all() and (rows[:, -1] == 7.0).all()


@pytest.mark.parametrize("hidden", [64, 90, 2304])
def test_norm_adds_an_unrounded_delta(ops, hidden):
    t = 9
    res, delta, w = rnd((t, hidden), 1), rnd((t, hidden), 2), rnd((hidden,), 3) + 1.0
    ref = f64(res) + f64(delta)
    r = res.clone().cuda()
    got = ops.rmsnorm(r, w.cuda(), 1e-5, torch.bfloat16, delta=delta.cuda(), write_back=True)
    assert rel(f64(r), ref) <= 1e-6 and rel(f64(got), plain.rms_norm(ref, f64(w), 1e-5)) <= 2.0 ** -8


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width, rows", [(48, 1), (48, 30), (256, 5), (512, 20), (512, 64), (90, 7), (264, 130)])
def test_entrance_of_a_pass(ops, dtype, width, rows):
    """x <- W [x; x0] + step[number] in front of a norm, the stream with and without a pending output; two entrances in a
    row read the same x0."""
    from from_scratch_inference_engine_amd.parts import HiddenState, OriginMix, RMSNorm

    eps = 1e-4
    part = OriginMix(width, 3)
    w = {"loop.in": rnd((width, 2 * width), 1, (2 * width) ** -0.5).to(dtype), "loop.step": rnd((3, width), 2)}
    part.weight, part.step = w["loop.in"].cuda(), w["loop.step"].cuda()
    part.prepare("cuda", dtype)
    norm, post = RMSNorm(width, eps), RMSNorm(width, eps)
    norm.weight, post.weight = (rnd((width,), 3) + 1.0).cuda(), (rnd((width,), 4) + 1.0).cuda()
    x0, y = rnd((rows, width), 5).to(dtype).float(), rnd((rows, width), 6).to(dtype)
    wn = {k: f64(v) for k, v in w.items()}
    for sums in (False, True):
        ctx = SimpleNamespace(compute_dtype=dtype, memo={}, partial_sums_ok=sums)
        hidden = HiddenState(x0.clone().cuda())
        part.begin(hidden, ctx)
        hidden.delta, hidden.delta_norm = y.cuda(), post
        part.forward(hidden, ctx, 2)
        got = norm(hidden, dtype)
        x = plain.enter_pass(f64(x0) + plain.rms_norm(f64(y), f64(post.weight), eps), f64(x0), wn, 2)
        assert rel(f64(hidden.residual), x) <= tol(dtype, 2e-6, 2.0 ** -7)
        assert rel(f64(got), plain.rms_norm(x, f64(norm.weight), eps)) <= tol(dtype, 5e-6)
        part.forward(hidden, ctx, 0)  # nothing pending
        norm(hidden, dtype)
        assert rel(f64(hidden.residual), plain.enter_pass(x, f64(x0), wn, 0)) <= tol(dtype, 5e-6, 2.0 ** -6)
    hidden.delta2 = y.cuda()
    with pytest.raises(RuntimeError, match="second pending"):
        part.forward(hidden, ctx, 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("t, heads, k, n, rot, pairs", [(5, 3, 8, 9, 6, 3), (16, 2, 40, 64, 8, -4), (17, 1, 64, 200, 16, 8), (100, 5, 96, 300, 4, -2),
                                                        (33, 2, 24, 17, 12, -4), (130, 3, 64, 128, 32, 16), (70, 2, 32, 60, 0, 0), (97, 4, 64, 192, 64, -32),
                                                        (129, 2, 40, 60, 8, 4), (161, 2, 64, 192, 16, -8), (300, 2, 72, 100, 10, 5)])
def test_product_per_head_with_gates_and_turned_parts(ops, dtype, t, heads, k, n, rot, pairs):
    """A factor a head, a gate for every output, both, none; the rotated runs of every head beside the product, zeros
    behind them; the columns in between stay.  Rows that allow 8-byte stores and rows that do not."""
    for x_off, x_gap, out_off, gap, g_off in ((16, 8, 8, 4, 8), (16, 8, 3, 2, 5), (1, 3, 0, 0, 0)):
        x_hs, pad = k + rot + x_gap, 6
        out_hs = n + gap + rot + pad
        x = rnd((t, x_off + heads * x_hs + 8), t).to(dtype)
        w = rnd((heads, n, k), n, k ** -0.5).to(dtype)
        gate, logits = torch.sigmoid(rnd((t, heads), 3)), rnd((t, g_off + heads * n), 4, 2.0).to(dtype)
        pos = np.arange(t) * 7 + 3
        turn = None
        if rot:
            f = 300.0 ** (-np.arange(abs(pairs)) / abs(pairs))
            table = torch.tensor(np.stack([np.cos(pos[:, None] * f), np.sin(pos[:, None] * f)], -1), dtype=torch.float32).cuda()
            turn = (k, n + gap, rot, pairs, rot + pad, table)
        xs = f64(x)[:, x_off:x_off + heads * x_hs].reshape(t, heads, x_hs)
        ref = np.einsum("thk,hnk->thn", xs[..., :k], f64(w))
        for g, gr in ((None, None), (gate, None), (None, logits), (gate, logits)):
            out = torch.full((t, out_off + heads * out_hs), 5.0, dtype=dtype).cuda()
            ops.head_gemm(x.cuda(), x_off, x_hs, w.cuda(), out, out_off, out_hs, gate=None if g is None else g.cuda(),
                          gate_rows=None if gr is None else gr.cuda()[:, g_off:], turn=turn)
            want = ref * (1.0 if g is None else f64(g)[:, :, None])
            if gr is not None:
                want = want * plain.sigmoid(f64(gr)[:, g_off:]).reshape(t, heads, n)
            got = f64(out)[:, out_off:].reshape(t, heads, out_hs)
            assert rel(got[..., :n], want) <= tol(dtype, 1e-5, 2.0 ** -7)
            assert (got[..., n:n + gap] == 5.0).all() and (f64(out)[:, :out_off] == 5.0).all()
            if rot:
                part = xs[..., k:k + rot].copy()
                turned = plain.rotate(part[..., :2 * abs(pairs)], pos, 300.0, pairs > 0)
                assert rel(got[..., n + gap:n + gap + 2 * abs(pairs)], turned) <= tol(dtype, 1e-5, 2.0 ** -7)
                assert np.array_equal(got[..., n + gap + 2 * abs(pairs):n + gap + rot], part[..., 2 * abs(pairs):])
                assert (got[..., n + gap + rot:] == 0.0).all()
            else:
                assert (got[..., n:] == 5.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_rows_without_a_query_latent(ops, dtype):
    """The cache rows and the gates are the same whether the projection holds a query latent or not."""
    t, q_rank, kv_rank, rot, heads, page, width, eps = 9, 24, 20, 6, 3, 4, 32, 1e-4
    proj = rnd((t, q_rank + kv_rank + rot + heads), 1, 2.0).to(dtype).cuda()
    wq, wkv = (rnd((q_rank,), 2) + 1.0).cuda(), (rnd((kv_rank,), 3) + 1.0).cuda()
    table = ops.rope_table(torch.arange(5, 5 + t, dtype=torch.int32).cuda(), torch.tensor([1.0, 0.2, 0.03], dtype=torch.float64).cuda())
    pools = []
    for rank in (q_rank, 0):
        k_pool, v_pool = (torch.zeros(s, dtype=dtype).cuda() for s in ((5, 1, page, width), (5, 1, width, page)))
        cq, gate = ops.latent_prep(proj, 0, rank, q_rank, kv_rank, rot, -3, q_rank + kv_rank + rot, heads, wq if rank else None, wkv, eps,
                                   table, slots=torch.arange(4, 4 + t, dtype=torch.int32).cuda(), k_pool=k_pool, v_pool=v_pool)
        assert cq.shape == (t, rank)
        pools.append((k_pool, v_pool, gate))
    assert all(torch.equal(a, b) for a, b in zip(*pools)) and pools[0][0].abs().sum() > 0
    c = plain.rms_norm(f64(proj)[:, q_rank:q_rank + kv_rank], f64(wkv), eps)
    assert rel(f64(pools[1][0]).reshape(-1, width)[4:4 + t, :kv_rank], c) <= tol(dtype, 5e-6, 2.0 ** -7)


# ------------------------------------------------------------------------------------------------
# whole models
# ------------------------------------------------------------------------------------------------
def mix(kind, heads, dim, rot, vdim, kv_rank, scale, base, q_rank=None, window=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": {"base": base, "dims": rot}}
    if kind != 1:
        m["q_rank"] = q_rank
    if kind == 2:
        m["mask"] = {"size": window}
    return {"type": "latent_attention" + ("" if kind == 1 else f"_{kind}"), "mixer": m}


def moe(ff, experts, top, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            **({"shared": {"ff": shared}} if shared else {})}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


# every kind of layer inside a loop of three passes; sizes that divide nothing
CONFIG_A = {"architecture": "Nenizen", "width": 72, "vocab": 91, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.5}, "logit_softcap": 9.0,
            "loop": {"start": 1, "stop": 4, "times": 3}, "layers": [
                layer(mix(2, 3, 20, 10, 14, 26, 0.35, 300.0, q_rank=33, window=11), dense(52, 0.8)),
                layer(mix(1, 4, 12, 6, 10, 30, 0.45, 50.0), moe(22, 6, 2, 34)),
                layer(mix(3, 2, 24, 4, 30, 18, 0.3, 1000.0, q_rank=20), dense(36, 1.7)),
                layer(mix(2, 5, 8, 12, 6, 40, 0.5, 80.0, q_rank=17, window=40), moe(30, 5, 3, None)),
                layer(mix(3, 3, 10, 8, 22, 28, 0.4, 9000.0, q_rank=50), None)]}
# a loop over all layers that runs once, another whose first layer is the model's first; no cap; one head; windows of one
# position and beyond every request; a query latent wider than the model
CONFIG_B = {"architecture": "Nenizen", "width": 48, "vocab": 64, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "loop": {"start": 0, "stop": 3, "times": 1}, "layers": [
                layer(mix(1, 1, 16, 16, 24, 32, 0.4, 1e4), dense(40, 2.0)),
                layer(mix(2, 2, 16, 2, 8, 14, 0.6, 20.0, q_rank=64, window=1), moe(16, 1, 1, 16)),
                layer(mix(2, 3, 12, 4, 9, 48, 0.3, 100.0, q_rank=24, window=500), None)]}
CONFIG_C = {"architecture": "Nenizen", "width": 64, "vocab": 120, "norm": {"eps": 1e-3}, "embedding": {"scale": 0.3}, "logit_softcap": 25.0,
            "loop": {"start": 0, "stop": 1, "times": 4}, "layers": [
                layer(mix(3, 6, 16, 0, 16, 32, 0.5, 10.0, q_rank=16), moe(24, 7, 7, 8)),
                layer(mix(1, 2, 8, 24, 40, 24, 0.4, 500.0), dense(32, 0.3))]}
# multiples of sixteen: the matrix-core kernels throughout, more heads than a tile of queries holds; no loop
CONFIG_D = {"architecture": "Nenizen", "width": 256, "vocab": 200, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.5}, "logit_softcap": 20.0,
            "layers": [
                layer(mix(1, 20, 32, 16, 48, 144, 0.3, 1e5), moe(64, 12, 5, 96)),
                layer(mix(2, 8, 64, 32, 64, 96, 0.25, 2e4, q_rank=128, window=33), dense(320, 1.2)),
                layer(mix(3, 4, 48, 16, 80, 112, 0.3, 700.0, q_rank=64), dense(128, 5.0))]}
# cache rows of more than 256 values
CONFIG_E = {"architecture": "Nenizen", "width": 96, "vocab": 70, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
            "loop": {"start": 0, "stop": 2, "times": 2}, "layers": [
                layer(mix(1, 3, 24, 18, 20, 270, 0.3, 1e4), dense(48, 1.0)),
                layer(mix(2, 2, 16, 8, 24, 300, 0.4, 300.0, q_rank=40, window=20), moe(20, 4, 2, 20))]}
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D, "E": CONFIG_E}


def nenizen_tensors(cfg, seed, sharp=True):
    """``sharp``: norms of the latents wide enough for peaked softmax rows (float32: a key that is missed shows at once).
    Not sharp: milder ones, for bfloat16, where a peaked row turns a rounding of the input into another key."""
    g = torch.Generator().manual_seed(seed)
    w = cfg["width"]

    def mat(rows, cols, gain=1.0):
        return torch.randn((rows, cols), generator=g) * (gain / math.sqrt(cols))

    def vec(n, centre, spread):
        return centre + torch.randn((n,), generator=g) * spread
    out = {"embed": torch.randn((cfg["vocab"], w), generator=g), "final.norm": vec(w, 1.0, 0.2)}
    if cfg.get("loop"):
        out.update({"loop.in": mat(w, 2 * w, 1.4), "loop.step": torch.randn((cfg["loop"]["times"], w), generator=g) * 0.8})

    def gated(p, ff):
        out.update({p + "gate": mat(ff, w, 1.5), p + "up": mat(ff, w, 1.5), p + "down": mat(w, ff, 1.5)})
    for i, lay in enumerate(cfg["layers"]):
        m, p, kind = lay["mixer"], f"l{i}.mix.", plain.KINDS[lay["type"]]
        h, d, r, e, c = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        size = 1.6 if sharp else 0.9
        out.update({f"l{i}.norm1": vec(w, 1.0, 0.2), f"l{i}.norm1b": vec(w, 1.0, 0.3)})
        if kind["latent_q"]:
            out.update({p + "dq": mat(m["q_rank"], w), p + "dq.norm": vec(m["q_rank"], size, 0.4), p + "uq": mat(h * (d + r), m["q_rank"])})
        else:
            out[p + "q"] = mat(h * (d + r), w, size)
        out.update({p + "dkv": mat(c + r, w), p + "dkv.norm": vec(c, size, 0.4), p + "uk": mat(h * d, c), p + "uv": mat(h * e, c),
                    p + "o": mat(w, h * e)})
        if kind["sink"]:
            out[p + "sink"] = vec(h, 0.5, 1.5)
        if kind["gate"]:
            out[p + "g"] = mat(h if kind["gate"] == "heads" else h * e, w, 2.0)
        mlp = lay["mlp"]
        if mlp is None:
            continue
        q = f"l{i}.mlp."
        out.update({f"l{i}.norm2": vec(w, 1.0, 0.2), f"l{i}.norm2b": vec(w, 1.0, 0.3)})
        if mlp["kind"] == "dense":
            gated(q, mlp["ff"])
        else:
            out[q + "router"] = mat(mlp["router"]["experts"], w, 4.0)
            for j in range(mlp["router"]["experts"]):
                gated(f"{q}e{j}.", mlp["expert"]["ff"])
            if mlp.get("shared"):
                gated(q + "shared.", mlp["shared"]["ff"])
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("nenizen")
    out = {}
    for name, cfg in CONFIGS.items():
        for tag, sharp in (("", True), ("~", False)):
            d = helpers.make_model_dir(root / (name + tag), cfg if sharp else without_choices(cfg), 0,
                                       tensors=nenizen_tensors(cfg, seed=ord(name), sharp=sharp))
            out[name + tag] = (d, plain.read_config(d), plain.read_weights(d))
    return out


def without_choices(cfg):
    """The same configuration with every expert chosen: the weights are then a continuous function of the input.  For whole
    models in bfloat16, where a choice made by a hair falls either way and the other expert is another function; the
    choice itself is tested alone in both types and in whole models in float32."""
    cfg = copy.deepcopy(cfg)
    for lay in cfg["layers"]:
        if lay["mlp"] is not None and lay["mlp"]["kind"] == "moe":
            lay["mlp"]["router"]["top"] = lay["mlp"]["router"]["experts"]
    return cfg


def close_enough(got, ref, dtype, what):
    """float32: 1e-4 of the largest logit at every position.  bfloat16: the root mean square of the difference against that
    of the logits, position by position."""
    got, ref = np.asarray(got, dtype=np.float64), np.asarray(ref, dtype=np.float64)
    assert got.shape == ref.shape and np.isfinite(got).all(), what
    if dtype == "float32":
        bad = np.abs(got - ref).max(-1) > 1e-4 * np.abs(ref).max()
        assert not bad.any(), f"{what}: first wrong position {int(np.argmax(bad))}, {np.abs(got - ref).max():.3e}"
    else:
        err = np.sqrt(((got - ref) ** 2).mean(-1)) / np.sqrt((ref ** 2).mean())
        assert (err > 0.12).sum() <= len(err) // 10 and np.median(err) <= 0.05, \
            f"{what}: {int((err > 0.12).sum())} of {len(err)} rows far off, the median row by {np.median(err):.3f}"


def step_through(runner, plan, seqs):
    """``plan``: steps of [(request, tokens)]; returns {request: logits of all its positions}.  A request is
    opened at its first entry and closed after its last token."""
    from from_scratch_inference_engine_amd.engine.context import StepEntry

    fed, caches, got = {r: 0 for r in seqs}, {}, {r: [] for r in seqs}
    for step in plan:
        entries = []
        for r, n in step:
            if r not in caches:
                caches[r] = runner.manager.open(r)
            entries.append(StepEntry(caches[r], seqs[r][fed[r]:fed[r] + n], list(range(n))))
            fed[r] += n
        out = runner.step(entries).cpu().numpy()
        row = 0
        for (r, n) in step:
            got[r].append(out[row:row + n])
            row += n
            if fed[r] == len(seqs[r]):
                runner.manager.close(caches.pop(r))
        runner.manager.check_invariants()
    return {r: np.concatenate(v) for r, v in got.items() if v}


def portions(sizes, total):
    out, i = [], 0
    while sum(out) < total:
        out.append(min(sizes[i % len(sizes)], total - sum(out)))
        i += 1
    return out


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_whole_in_portions_decoded_and_batched(models, name, dtype):
    """The same requests whole, token by token (through the captured decode graphs), in portions down to two tokens
    and one, and in batches of unequal requests that start and end at different steps in a pool so small that pages
    and slots are taken again."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models[name if dtype == "float32" else name + "~"]
    vocab = cfg["vocab"]
    seqs = {"a": helpers.token_ids(vocab, 75, 1), "b": helpers.token_ids(vocab, 1, 2), "c": helpers.token_ids(vocab, 33, 3),
            "d": helpers.token_ids(vocab, 130, 4), "e": helpers.token_ids(vocab, 18, 5)}
    ref = {r: plain.forward(cfg, w, ids) for r, ids in seqs.items()}
    runner = Runner(load_model(d, dtype=dtype), page_size=8, num_pages=40, max_requests=3)
    assert runner.graphs.enabled

    def check(got, r, what):
        close_enough(got[r], ref[r], dtype, what)
    got = step_through(runner, [[(r, len(ids))] for r, ids in seqs.items()], seqs)
    whole = got
    for r in seqs:
        check(got, r, f"{name} whole {r}")
    for r, head in (("a", 10), ("c", 1)):
        got = step_through(runner, [[(r, head)]] + [[(r, 1)]] * (len(seqs[r]) - head), {r: seqs[r]})
        check(got, r, f"{name} decode {r}")
    assert runner.graphs.replays > 50
    for sizes in ([2, 7, 1, 16, 3, 2, 33, 8, 64], [2], [9, 40]):
        got = step_through(runner, [[("d", n)] for n in portions(sizes, len(seqs["d"]))], {"d": seqs["d"]})
        check(got, "d", f"{name} portions {sizes}")
    plan = [[("a", 30), ("c", 2), ("b", 1)], [("a", 1), ("c", 20), ("e", 3)], [("c", 11), ("a", 44), ("e", 1)],
            [("e", 14), ("d", 9)], [("d", 120)], [("d", 1)]]
    got = step_through(runner, plan, seqs)
    for r in seqs:
        check(got, r, f"{name} batched {r}")
        if dtype == "float32":
            close_enough(got[r], whole[r], dtype, f"{name} batched against alone {r}")
    assert all(a.pages_issued_again() for a in runner.manager.allocators)


# ---- keys that must and must not be seen
def loud_pair(cfg, tensors, query, key, gain):
    """Adds to a one-layer model's W_uk, head by head, what gives token ``query``'s scores with token ``key`` ``gain`` more
    (before the rotated parts' share): a rank-one matrix along the head's query and the key's latent."""
    lay, eps, p = cfg["layers"][0], cfg["norm"]["eps"], "l0.mix."
    m, kind = lay["mixer"], plain.KINDS[lay["type"]]
    w = {k: v.double().numpy() for k, v in tensors.items()}
    h = plain.rms_norm(w["embed"][[query, key]] * cfg["embedding"]["scale"], w["l0.norm1"], eps)
    q = plain.rms_norm(h[:1] @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T if kind["latent_q"] else h[:1] @ w[p + "q"].T
    q = q.reshape(m["heads"], -1)[:, :m["dim"]]
    c = plain.rms_norm(h[1] @ w[p + "dkv"].T[:, :m["kv_rank"]], w[p + "dkv.norm"], eps)
    uk = w[p + "uk"].reshape(m["heads"], m["dim"], -1)
    uk = uk + gain / m["scale"] * (q / (q * q).sum(-1, keepdims=True))[:, :, None] * (c / (c * c).sum())[None, None, :]
    return {**tensors, p + "uk": torch.from_numpy(uk.reshape(-1, m["kv_rank"])).to(torch.bfloat16).contiguous()}


SINGLE = {"values": mix(1, 3, 32, 8, 24, 56, 0.15, 1e4), "window": mix(2, 2, 32, 16, 24, 64, 0.15, 1e4, q_rank=40, window=37),
          "sink": mix(3, 3, 32, 16, 24, 48, 0.15, 1e4, q_rank=40)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_one_loud_key_among_hundreds(tmp_path, name, dtype):
    """One layer; a query whose score with one key stands out by far.  The key lies at the request's first position, at
    page borders, far away, at the query's own place minus one, just inside and just outside the window; the query
    comes in a prompt, at the start of a portion, and as a decoded token.  That the key is seen (or not) is first
    shown on the plain model: without it the logits are others (the same)."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    vocab, query, key = 60, 58, 59
    cfg = {"architecture": "Nenizen", "width": 64, "vocab": vocab, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.5},
           "layers": [layer(SINGLE[name], None)]}
    tensors = loud_pair(cfg, nenizen_tensors(cfg, 5, sharp=False), query, key, 14.0)
    tensors["l0.norm1b"] = tensors["l0.norm1b"] * 4.0  # (the layer's output weighs more than the embedding it is added to)
    d = helpers.make_model_dir(tmp_path / name, cfg, 0, tensors=tensors)
    cfg, w = plain.load(d)
    window = cfg["layers"][0]["mixer"].get("mask", {}).get("size")
    page = 8
    runner = Runner(load_model(d, dtype=dtype), page_size=page, num_pages=90, max_requests=2)
    cases = [(0, 1), (0, 300), (7, 255), (8, 256), (15, 16), (40, 90), (63, 64), (1, 600)]
    if window:
        cases += [(p, p + dist) for p in (0, 7, 8, 33) for dist in (window - 1, window, window + 1)]
    seen_any = unseen_any = False
    for at, q_at in cases:
        ids = [t % (vocab - 2) for t in helpers.token_ids(vocab, q_at + 1, 31 + at)]
        ids[q_at], ids[at] = query, key
        ref = plain.forward(cfg, w, ids)
        other = plain.forward(cfg, w, ids[:at] + [ids[at] // 3] + ids[at + 1:])
        moved = np.abs(ref[-1] - other[-1]).max() / np.abs(ref).max()
        seen = not window or q_at - at < window
        assert moved > 0.15 if seen else moved == 0.0, (at, q_at, moved)
        seen_any, unseen_any = seen_any or seen, unseen_any or not seen
        n = q_at + 1
        for plan in ([[("r", n)]], [[("r", n - 1)], [("r", 1)]], [[("r", n - n // 2)], [("r", n // 2)]] if n > 1 else [[("r", 1)]]):
            got = step_through(runner, plan, {"r": ids})["r"]
            if dtype == "float32":
                close_enough(got, ref, dtype, f"{name} key {at} query {q_at}")
            else:
                err = np.abs(got[-1] - ref[-1]).max() / np.abs(ref).max()
                assert err <= 0.05, (name, at, q_at, err)
    assert seen_any and (unseen_any or not window)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_sink_that_takes_most_of_the_weight(tmp_path, dtype):
    """The first tokens of a request under sinks from far below to far above their scores: at position 0 the output is
    1 / (1 + exp(sink - score)) of the value, not the value."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    cfg = {"architecture": "Nenizen", "width": 64, "vocab": 60, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.5},
           "layers": [layer(mix(3, 5, 32, 16, 24, 48, 0.1, 1e4, q_rank=40), None)]}
    tensors = nenizen_tensors(cfg, 7, sharp=False)
    tensors["l0.norm1b"] = tensors["l0.norm1b"] * 4.0
    tensors["l0.mix.sink"] = torch.tensor([-20.0, -1.0, 1.0, 3.0, 6.0]).bfloat16()
    d = helpers.make_model_dir(tmp_path / "m", cfg, 0, tensors=tensors)
    cfg, w = plain.load(d)
    ids = helpers.token_ids(60, 40, 3)
    ref = plain.forward(cfg, w, ids)
    bare = plain.forward(cfg, {**w, "l0.mix.sink": w["l0.mix.sink"] * 0 - 100.0}, ids)
    assert np.abs(ref - bare).max(-1).min() > 0.05 * np.abs(ref).max()
    runner = Runner(load_model(d, dtype=dtype), page_size=8, num_pages=40, max_requests=2)
    for plan in ([[("r", 40)]], [[("r", 1)]] * 40, [[("r", 2)]] * 20):
        got = step_through(runner, plan, {"r": ids})["r"]
        close_enough(got, ref, dtype, "sinks")


def test_long_decoding(models):
    """Four hundred decoded tokens in float32, page after page, windows handing their pages back in every pass."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models["A"]
    ids = helpers.token_ids(cfg["vocab"], 405, 11)
    ref = plain.forward(cfg, w, ids)
    runner = Runner(load_model(d, dtype="float32"), page_size=8, num_pages=60, max_requests=1)
    got = step_through(runner, [[("a", 5)]] + [[("a", 1)]] * 400, {"a": ids})
    close_enough(got["a"], ref, "float32", "long decode")


def test_passes_keep_caches_of_their_own(models):
    """A model of three passes keeps three caches a looped layer, and the pools of one geometry hold a plane for each."""
    from from_scratch_inference_engine_amd import load_model

    d, cfg, _ = models["A"]
    model = load_model(d, dtype="float32")
    assert sum(len(ids) for ids in model.cache_layout.group_caches) == 2 + 3 * 3
    assert model.call_cache == list(range(11))


@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_greedy_generation_through_the_engine(models, name):
    """Prompts of unequal length generated together through the LLM entry point and its scheduler (three at a
    time, portions of at most 16 tokens), in float32: the tokens are the plain implementation's greedy ones."""
    from from_scratch_inference_engine_amd import GenerationConfig, LLM

    d, cfg, w = models[name]
    prompts = [helpers.token_ids(cfg["vocab"], n, 20 + n) for n in (1, 9, 40, 23)]
    n_new = 40
    llm = LLM(d, dtype="float32", block_size=8, num_blocks=64, max_batch=3, eos_id=-1, prefill_chunk=16)
    got = llm.generate_ids_batch(prompts, GenerationConfig(max_tokens=n_new))
    for prompt, mine in zip(prompts, got):
        assert len(mine) == n_new
        logits = plain.forward(cfg, w, prompt + mine)[len(prompt) - 1:-1]
        for i, tok in enumerate(mine):  # the plain choice, unless the two best are a rounding apart
            assert tok == int(logits[i].argmax()) or (logits[i].max() - logits[i, tok]) <= 1e-4 * np.abs(logits).max(), (len(prompt), i)
    assert llm.engine.runner.graphs.replays > 0


@pytest.mark.parametrize("name", ["A", "C"])
def test_replay_program_runs_the_model(models, tmp_path, name):
    """bin/trace_run on the architecture: a prompt in portions beside another request's single tokens, then a third
    request in the slot and pages that the second gave back."""
    d, cfg, w = models[name]
    a, b, c = (helpers.token_ids(cfg["vocab"], n, 7 + n) for n in (50, 20, 9))
    tb = helpers.TraceBuilder()
    tb.step([("a", a[:17], [16]), ("b", b[:1], [0])])
    for i in range(1, 20):
        lo, hi = 17 + (i - 1) * 2, min(50, 17 + i * 2)
        entries = [("b", b[i:i + 1], [0])] + ([("a", a[lo:hi], list(range(hi - lo)))] if lo < 50 else [])
        tb.step(entries, end=["b"] if i == 19 else [])
    tb.step([("c", c, list(range(9)))], end=["a", "c"])
    for dtype in ("float32", "bfloat16"):
        d, cfg, w = models[name if dtype == "float32" else name + "~"]
        per = helpers.collect(tb, helpers.run_trace(d, dtype, tb.steps, 128, tmp_path / dtype))
        for rid, ids in (("a", a), ("b", b), ("c", c)):
            ref = plain.forward(cfg, w, ids)
            pos = sorted(per[rid])
            close_enough(np.stack([per[rid][p] for p in pos]), ref[pos], dtype, f"replay {rid}")


WIDE = {"architecture": "Nenizen", "width": 2048, "vocab": 300, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0}, "logit_softcap": 30.0,
        "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [
            layer(mix(3, 8, 64, 32, 128, 160, 0.15, 1e4, q_rank=512), dense(3072, 1.5)),
            layer(mix(1, 8, 64, 64, 64, 192, 0.15, 1e4), moe(256, 4, 4, 512)),
            layer(mix(2, 16, 32, 32, 64, 96, 0.2, 1e4, q_rank=256, window=24), dense(2048, 0.9))]}


@pytest.mark.parametrize("copies", [True, False])
def test_a_model_wide_enough_for_the_fused_steps(tmp_path, copies):
    """Matrices large enough for fragment-ordered copies and for products that leave partial sums: decode steps of one to
    seventy requests, a prompt, portions, in bfloat16, with and without the copies."""
    from from_scratch_inference_engine_amd.engine.context import StepEntry
    from from_scratch_inference_engine_amd.engine.model import Model, Runner

    d = helpers.make_model_dir(tmp_path / "wide", WIDE, 0, tensors=nenizen_tensors(WIDE, 3, sharp=False))
    cfg, w = plain.load(d)
    w = {k: v.astype(np.float32) for k, v in w.items()}  # (the oracle in float32: its rounding is nothing beside bfloat16's)
    model = Model.from_pretrained(d, dtype="bfloat16", weight_copies=copies)
    assert (model.entrances[0].linear.streamed is not None) == copies
    runner = Runner(model, page_size=16, num_pages=160, max_requests=72)
    ids = helpers.token_ids(300, 48, 1)
    ref = plain.forward(cfg, w, ids)
    for plan in ([[("r", 48)]], [[("r", 20)], [("r", 2)], [("r", 17)]] + [[("r", 1)]] * 9):
        close_enough(step_through(runner, plan, {"r": ids})["r"], ref, "bfloat16", f"wide {len(plan)}")
    distinct = [helpers.token_ids(300, 4, 50 + i) for i in range(6)]
    refs = [plain.forward(cfg, w, s) for s in distinct]
    for batch in (1, 3, 9, 20, 40, 70):
        caches = [runner.manager.open(i) for i in range(batch)]
        runner.step([StepEntry(c, distinct[i % 6][:3], []) for i, c in enumerate(caches)])
        got = runner.step([StepEntry(c, distinct[i % 6][3:], [0]) for i, c in enumerate(caches)]).cpu().numpy()
        close_enough(got, np.stack([refs[i % 6][3] for i in range(batch)]), "bfloat16", f"wide batch {batch}")
        for c in caches:
            runner.manager.close(c)


def test_command_line_writes_a_random_model_and_generates(tmp_path):
    """random-model from a config.json, then generate from that folder and, without a folder, from the configuration
    and the seed: the architecture is served by the same command line as the others."""
    (tmp_path / "cfg.json").write_text(json.dumps(CONFIG_A))
    env = dict(os.environ, PYTHONPATH=str(helpers.ROOT))
    base = [sys.executable, "-m", "from_scratch_inference_engine_amd"]
    made = subprocess.run(base + ["random-model", "--config", str(tmp_path / "cfg.json"), "--out", str(tmp_path / "m"), "--seed", "5"],
                          capture_output=True, text=True, env=env, timeout=300)
    assert made.returncode == 0, made.stderr[-2000:]
    common = ["--prompt-ids", "3 1 4 1 5 9 2 6", "--max-tokens", "12", "--num-blocks", "64", "--max-batch", "4", "--dtype", "float32"]
    a = subprocess.run(base + ["generate", "--model-dir", str(tmp_path / "m")] + common, capture_output=True, text=True, env=env, timeout=300)
    b = subprocess.run(base + ["generate", "--config", str(tmp_path / "cfg.json"), "--random-weights", "5"] + common,
                       capture_output=True, text=True, env=env, timeout=300)
    assert a.returncode == 0 and b.returncode == 0, a.stderr[-2000:] + b.stderr[-2000:]
    tokens = a.stdout.strip().splitlines()[-1].split()
    assert len(tokens) == 12 and all(0 <= int(t) < CONFIG_A["vocab"] for t in tokens)
    cfg, w = plain.read_config(tmp_path / "m"), plain.read_weights(tmp_path / "m")
    ids = [3, 1, 4, 1, 5, 9, 2, 6] + [int(t) for t in tokens]
    logits = plain.forward(cfg, w, ids)[7:-1]
    for i, t in enumerate(tokens):
        assert int(t) == int(logits[i].argmax()) or (logits[i].max() - logits[i, int(t)]) <= 1e-4 * np.abs(logits).max(), i
    assert len(b.stdout.strip().splitlines()[-1].split()) == 12
