"""Romepel on the GPU against the plain implementation (plain_romepel.py): every mechanism alone, then whole models of
small configurations through the step function, the scheduler and the replay.

The weights are drawn here with a spread that keeps activations of order one (standard deviation fan_in^-1/2; biases,
position vectors, decay biases and the norms' offsets wide, queries and keys loud), so that softmax rows are peaked and a
position, a bias or a window's edge that is wrong shows."""

import copy
import json
import math
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
import plain_romepel as plain


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
    got, ref = torch.as_tensor(got, dtype=torch.float64), torch.as_tensor(ref, dtype=torch.float64)
    return ((got - ref).abs().max() / ref.abs().max().clamp_min(1e-30)).item()


def tol(dtype, f32=2e-5, bf16=2.0 ** -6):
    return f32 if dtype == torch.float32 else bf16


# ------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden, scale", [(64, 1.0), (1030, 0.5), (7, 1.0)])
def test_embedding_with_position_vectors(ops, dtype, hidden, scale):
    table, places = rnd((50, hidden), 1).to(dtype), rnd((33, hidden), 2, 3.0).to(dtype)
    ids = torch.tensor([3, 49, 0, 7, 7, 7], dtype=torch.int32)
    pos = torch.tensor([0, 32, 5, 5, 31, 1], dtype=torch.int32)
    ref = table.double()[ids.long()] * scale + places.double()[pos.long()]
    args = (table.cuda(), ids.cuda())
    got = ops.embedding(*args, scale=scale, pos_table=places.cuda(), positions=pos.cuda())
    assert got.dtype == torch.float32 and rel(got.cpu(), ref) <= 1e-6  # the stream is float32 in both precisions
    # rows that do not exist (a filler's positions may run past the table) count as zeros and read nothing
    ids[1], pos[2], pos[3] = 50, 33, -1
    got = ops.embedding(args[0], ids.cuda(), scale=scale, pos_table=places.cuda(), positions=pos.cuda()).cpu()
    ref[1], ref[2], ref[3] = places.double()[32], table.double()[0] * scale, table.double()[7] * scale
    assert rel(got, ref) <= 1e-6
    assert torch.equal(ops.embedding(args[0], args[1], scale=scale).cpu(), (args[0].float().cpu()[args[1].cpu().long()] * scale))


def test_query_temperature(ops):
    for coef, every in ((0.3, 8), (1.7, 1), (-0.2, 3), (0.5, 1000), (0.0, 5), (0.4, 2.5)):
        pos = torch.tensor([0, 1, 2, 6, 7, 8, 14, 15, 16, 998, 999, 1000, 1999, 123456], dtype=torch.int32)
        got = ops.query_temperature(pos.cuda(), coef, every).cpu()
        assert rel(got, plain.query_temperature(pos.tolist(), coef, every)) <= 1e-6, (coef, every)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("p, q", [(0.4, -0.7), (-30.0, 5.0), (25.0, -40.0)])
def test_activation_alone_and_in_the_products(ops, dtype, p, q):
    """xIELU with its bias: the kernel of its own, the one that adds partial sums, and the two products that have it in
    their epilogue; values near zero on both sides, where the two branches and the exponential's series meet."""
    act64 = torch.tensor([p, q], dtype=torch.float64)
    act = ops.PointAct("xielu", plain.softplus(act64[0]).item(), 0.5 + plain.softplus(act64[1]).item())
    special = torch.tensor([0.0, 1e-6, -1e-6, -1e-3, -0.1, -0.49, -0.5, -0.51, -1.0, -8.0, -100.0, 3.0])
    for rows, cols in ((5, 96), (3, 37), (2, 2056)):
        x, b = rnd((rows, cols), 1, 2.0), rnd((cols,), 2)
        x[:, :12], b[:12] = special, 0.0
        x = x.to(dtype)
        for bias in (b, None):
            z = x.double() + (0 if bias is None else b.double())
            ref = plain.xielu(z, act64)
            got = ops.bias_act(x.cuda(), None if bias is None else b.cuda(), act).float().cpu()
            # against the size of each argument and value themselves: the small ones are rounded, not lost
            err = (got.double() - ref).abs() / (ref.abs() + 0.1 * z.abs() + (1e-6 if dtype == torch.float32 else 1e-4))
            assert err.max().item() <= (1e-5 if dtype == torch.float32 else 2.0 ** -7), (rows, cols)
    if dtype == torch.bfloat16:
        parts, b = rnd((3, 6, 40), 3), rnd((40,), 4)
        got = ops.sum_round(parts.cuda(), b.cuda(), act).float().cpu()
        assert rel(got, plain.xielu(parts.double().sum(0) + b.double(), act64)) <= 2.0 ** -7
        for m, n, k in ((1, 132, 256), (9, 200, 128), (16, 64, 384), (30, 132, 128), (64, 76, 256)):
            x, w, b = rnd((m, k), m).to(dtype), rnd((n, k), n, k ** -0.5).to(dtype), rnd((n,), k)
            ref = plain.xielu(x.double() @ w.double().t() + b.double(), act64)
            if m <= 16:
                assert rel(ops.gemm_mfma_skinny_act(x.cuda(), w.cuda(), b.cuda(), act).float().cpu(), ref) <= 2.0 ** -6
            assert ops.gemm_mfma_wide_act_takes(m, w)
            for weight in (w.cuda(), ops.fragment_order(w.cuda())):
                for shape in (dict(), dict(waves=4, blocks=1), dict(waves=8, blocks=2)):
                    assert rel(ops.gemm_mfma_wide_act(x.cuda(), weight, b.cuda(), act, **shape).float().cpu(), ref) <= 2.0 ** -6
        assert not ops.gemm_mfma_wide_act_takes(65, w) and not ops.gemm_mfma_wide_act_takes(4, w[:, :100])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden, n_parts", [(96, 0), (257, 3), (4100, 0), (1024, 8)])
def test_sandwich_norm_with_the_products_bias(ops, dtype, hidden, n_parts):
    """The bias of the sublayer's last product is added before the norm of its output."""
    t, res, delta, bias = 7, rnd((7, hidden), 1, 3.0), rnd((n_parts or 1, 7, hidden), 2, 0.5), rnd((hidden,), 5, 2.0)
    if dtype == torch.bfloat16 and not n_parts:
        delta = delta.bfloat16().float()
    wp, w = 1 + rnd((hidden,), 3, 0.3), 1 + rnd((hidden,), 4, 0.3)
    v = res.double() + plain.norm_plain_weight(delta.double().sum(0) + bias.double(), wp.double(), 1e-5)
    ref = plain.norm_plain_weight(v, w.double(), 1e-6)
    d_dev, r_dev = (delta if n_parts else delta[0].to(dtype)).cuda(), res.cuda().clone()
    args = (wp.cuda(), 1e-5, w.cuda(), 1e-6, dtype)
    out = ops.sandwich_norm(r_dev, d_dev, *args, write_back=True, delta_bias=bias.cuda())
    assert rel(out.float().cpu(), ref) <= tol(dtype, bf16=2.0 ** -7) and rel(r_dev.cpu(), v) <= 2e-6
    rows = torch.tensor([5, 0, 5, 2], dtype=torch.int32).cuda()
    out = ops.sandwich_norm(res.cuda(), d_dev, *args, rows=rows, delta_bias=bias.cuda())
    assert rel(out.float().cpu(), ref[rows.cpu().long()]) <= tol(dtype, bf16=2.0 ** -7)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("defer", [False, True])
def test_feed_forward_part(ops, dtype, defer, monkeypatch):
    """The part at row counts that take each of its ways (epilogue, partial sums, fragment-ordered copy, library), with
    its last bias added or left pending."""
    from from_scratch_inference_engine_amd.parts.base import make_part, prepare_parts
    from from_scratch_inference_engine_amd.parts.linear import Linear

    h, ff = 1024, 392
    up, up_b, down, down_b = rnd((ff, h), 1, h ** -0.5), rnd((ff,), 2), rnd((h, ff), 3, ff ** -0.5), rnd((h,), 4)
    up, down, act = up.to(dtype), down.to(dtype), torch.tensor([0.3, -0.6])
    for copies_from in (16 << 20, 0):
        monkeypatch.setattr(Linear, "streamed_copy_from", copies_from)
        ffn = make_part("feed_forward", "plain", hidden_size=h, intermediate_size=ff, defer_bias=defer)
        for name, t in (("up_weight", up), ("up_bias", up_b), ("down_weight", down), ("down_bias", down_b), ("act", act)):
            setattr(ffn, name, t.cuda())
        prepare_parts(ffn, torch.device("cuda:0"), dtype, {"weight_copies": True})
        assert (ffn.up.streamed is not None) == (dtype == torch.bfloat16 and copies_from == 0)
        for m in (1, 5, 16, 17, 40, 64, 90, 300):
            x = rnd((m, h), m).to(dtype)
            y = ffn.forward(x.cuda(), SimpleNamespace(partial_sums_ok=True)).float()
            y = (y.sum(0) if y.ndim == 3 else y).cpu()
            if defer:
                y = y + ffn.residual_bias.cpu()
            else:
                assert ffn.residual_bias is None
            ref = plain.dense_feed_forward(x.double(), up.double(), up_b.double(), act.double(), down.double(), down_b.double())
            assert rel(y, ref) <= tol(dtype), m


# attention ---------------------------------------------------------------------------------------
def scored(ops, case, heads, kv, hd, window, scale, slopes, factor, share_keys=True, softcap=None, sinks=None):
    from from_scratch_inference_engine_amd.parts.attention import paged_attention

    plan = {k: (torch.from_numpy(v).cuda() if isinstance(v, np.ndarray) else v) for k, v in case["plan"].items()}
    cache = SimpleNamespace(k_pool=case["k_pool"].cuda(), v_pool=case["v_pool"].cuda(), block_tables=case["tables"].cuda(),
                            page_size=case["k_pool"].shape[2])
    q = case["q"].cuda()
    dev = lambda t: None if t is None else t.float().cuda()
    return paged_attention(q, heads * hd, cache, SimpleNamespace(**plan), heads, kv, hd, window, scale, q.shape[0],
                           sinks=dev(sinks), share_keys=share_keys, softcap=softcap, slopes=dev(slopes), row_scale=dev(factor)).float().cpu()


def plain_rows(q, k, v, past, heads, kv, hd, window, scale, slopes, factor):
    n = q.shape[0]
    return plain.biased_attention(q.double().reshape(n, heads, hd), k.double().reshape(-1, kv, hd), v.double().reshape(-1, kv, hd),
                                  past, scale, window, slopes.double(), factor.double()).reshape(n, heads * hd)


@pytest.mark.parametrize("window", [None, 150, 33])
@pytest.mark.parametrize("dtype, scalar, heads, kv, hd", [
    (torch.float32, True, 6, 2, 24), (torch.float32, True, 3, 3, 50), (torch.bfloat16, True, 5, 1, 40),
    (torch.bfloat16, False, 6, 2, 64), (torch.bfloat16, False, 12, 1, 48), (torch.bfloat16, False, 3, 3, 128),
    (torch.bfloat16, False, 40, 1, 96), (torch.bfloat16, False, 2, 1, 160), (torch.bfloat16, False, 4, 2, 256)])
def test_attention_with_slopes_and_a_factor_a_token(ops, dtype, scalar, heads, kv, hd, window):
    """Every attention kernel: decodes cut into items and merged, short and long portions (through the kernel that shares
    keys and without it), first tokens; each alone (slopes, factor) and both."""
    from test_kernels_gpu import paged_case
    from from_scratch_inference_engine_amd.parts.attention import AttentionPlanner

    seqs, page, scale = [(0, 1), (0, 2), (700, 1), (0, 150), (300, 2), (123, 70), (1500, 1), (500, 100)], 16, 0.17
    slopes = plain.distance_slopes(heads)
    factors = [plain.query_temperature(range(p, p + n), 0.6, 50) for p, n in seqs]
    AttentionPlanner.compute_units = 4096  # as on an idle device: decodes are cut into many items and merged
    try:
        case = paged_case(seqs, heads, kv, hd, page, dtype, seed=hd, window=window, scalar=scalar)
    finally:
        AttentionPlanner.compute_units = None
    assert case["plan"]["mfma"] == (not scalar) and case["plan"]["n_large"] > 0
    for use_slopes, use_factor in ((True, True), (True, False), (False, True)):
        s = slopes if use_slopes else torch.zeros(heads, dtype=torch.float64)
        f = factors if use_factor else [torch.ones(n, dtype=torch.float64) for _, n in seqs]
        given = (slopes if use_slopes else None, torch.cat(factors) if use_factor else None)
        outs = [scored(ops, case, heads, kv, hd, window, scale, *given)]
        if not scalar and ops.attention_mfma_lds_ok(hd, page):
            outs.append(scored(ops, case, heads, kv, hd, window, scale, *given, share_keys=False))
        for out in outs:
            row = 0
            for (p, n), q, k, v, fac in zip(seqs, case["qs"], case["ks"], case["vs"], f):
                ref = plain_rows(q, k, v, p, heads, kv, hd, window, scale, s, fac)
                err = (out[row:row + n].double() - ref).abs().max().item()
                assert err <= (2e-5 if dtype == torch.float32 else 2.0 ** -7) * v.abs().max().item(), (p, n, use_slopes, use_factor, err)
                row += n


@pytest.mark.parametrize("dtype, scalar, hd", [(torch.float32, True, 32), (torch.bfloat16, True, 32), (torch.bfloat16, False, 48),
                                               (torch.bfloat16, False, 64), (torch.bfloat16, False, 128)])
def test_keys_at_the_windows_edges_far_away_and_at_page_borders(ops, dtype, scalar, hd):
    """Loud queries for which one key carries nearly the whole softmax although its distance costs it: the window's first
    key, keys on either side of a page's border, the query's own position; louder keys sit just outside the window and
    right after the query, where it must not look."""
    from test_kernels_gpu import paged_case

    heads, kv, page, window, scale = 4, 2, 16, 100, 0.5
    seqs = [(640, 1), (350, 3), (0, 140), (95, 8)]
    slopes = plain.distance_slopes(heads)  # up to 1/4: 25 off a key at the window's far end
    targets = {}

    def edit(qs, ks, vs):
        for s, (p, n) in enumerate(seqs):
            ks[s].mul_(0.02), qs[s].mul_(0.02)
            every = -(-n // (hd // 2))  # a direction of its own for every loud query
            for i in range(0, n, every):
                pos = p + i
                far = max(0, pos - window + 1)
                choice = (far, pos, pos - pos % page, max(far, pos - pos % page - 1))[i // every % 4]
                targets[s, i] = choice
                u = torch.zeros(hd)
                u[(3 * s + i // every) % hd] = 1.0
                # score 0.5 * 8 * 20 = 80; what lies outside would score twice that
                qs[s][i] += (8.0 * u).repeat(heads)
                for key, size in ((choice, 20.0), (pos + 1, 40.0), (pos - window, 40.0)):
                    if 0 <= key < p + n:
                        ks[s][key] += (size * u).repeat(kv)
            for t in (qs[s], ks[s]):
                t.copy_(t.to(dtype).float())
    case = paged_case(seqs, heads, kv, hd, page, dtype, seed=4, window=window, edit=edit, scalar=scalar)
    factor = [torch.ones(n, dtype=torch.float64) for _, n in seqs]
    row, found = 0, 0
    out = scored(ops, case, heads, kv, hd, window, scale, slopes, torch.cat(factor))
    for s, ((p, n), q, k, v) in enumerate(zip(seqs, case["qs"], case["ks"], case["vs"])):
        ref = plain_rows(q, k, v, p, heads, kv, hd, window, scale, slopes, factor[s])
        assert (out[row:row + n].double() - ref).abs().max() <= (3e-5 if dtype == torch.float32 else 2.0 ** -6) * v.abs().max()
        for i in [i for seq, i in targets if seq == s]:
            mine = v[targets[s, i]].reshape(kv, hd).repeat_interleave(heads // kv, 0).reshape(-1)
            assert (out[row + i] - mine).abs().max() <= 0.02 * v.abs().max(), (s, i)
            found += 1
        row += n
    assert found >= 25


@pytest.mark.parametrize("heads, kv, hd, window, units", [(8, 2, 64, None, 4096), (6, 2, 128, 60, 1), (5, 5, 32, 40, 4096), (16, 1, 96, None, 1)])
def test_attention_from_the_products_sums_without_rotation(ops, heads, kv, hd, window, units):
    """A decode step in one kernel from the q/k/v product's partial sums (no table: nothing turns), with slopes and a
    factor a token, against the same steps one after the other; and the pools they leave."""
    from test_kernels_gpu import paged_case
    from from_scratch_inference_engine_amd.parts.attention import AttentionPlanner

    page, pasts, n_parts = 16, [0, 5, 31, 32, 300, 700, 1023], 3
    AttentionPlanner.compute_units = units
    try:
        case = paged_case([(p, 1) for p in pasts], heads, kv, hd, page, torch.bfloat16, seed=9, window=window)
    finally:
        AttentionPlanner.compute_units = None
    plan, t, width = case["plan"], len(pasts), (heads + 2 * kv) * hd
    parts, b = rnd((n_parts, t, width), 5).cuda(), rnd((width,), 6).cuda()
    positions = torch.tensor(pasts, dtype=torch.int32).cuda()
    tables = case["tables"]
    slots = torch.tensor([int(tables[s, p // page]) * page + p % page for s, p in enumerate(pasts)], dtype=torch.int32).cuda()
    items, merges = torch.from_numpy(plan["items"]).cuda(), torch.from_numpy(plan["merges"]).cuda()
    bias = dict(slopes=plain.distance_slopes(heads).float().cuda(), row_scale=ops.query_temperature(positions, 0.7, 20))
    pools = lambda: (case["k_pool"].cuda().clone(), case["v_pool"].cuda().clone(), tables.cuda())
    records = lambda: torch.zeros(max(plan["n_partial"], 1) * heads * (hd + 2)).cuda()
    k1, v1, bt = pools()
    qkv = torch.empty(t, width, dtype=torch.bfloat16).cuda()
    ops.rope_kv_write(qkv, positions, heads, kv, hd, None, slots=slots, k_pool=k1, v_pool=v1, page_size=page, bias=b, parts=parts,
                      by_rows=True)
    whole = (parts.double().sum(0) + b.double()).cpu()
    assert rel(qkv[:, :heads * hd].float().cpu(), whole[:, :heads * hd]) <= 2.0 ** -8
    out1, rec1 = torch.zeros(t, heads * hd, dtype=torch.bfloat16).cuda(), records()
    ops.attention_mfma(qkv, width, k1, v1, bt, items, plan["n_small"], out1, rec1, heads, kv, hd, window, 0.2, t, large=False,
                       waves=plan["waves"], **bias)
    k2, v2, bt = pools()
    out2, rec2 = torch.zeros_like(out1), records()
    ops.attention_mfma_qkv(parts, b, None, slots, k2, v2, bt, items, plan["n_small"], out2, rec2, heads, kv, hd, window, 0.2,
                           waves=plan["waves"], **bias)
    if plan["n_merges"]:
        ops.attention_merge(rec1, merges, plan["n_merges"], out1, heads, hd)
        ops.attention_merge(rec2, merges, plan["n_merges"], out2, heads, hd)
    assert torch.equal(k1, k2) and torch.equal(v1, v2)  # nothing is rotated: the same sums, rounded once
    for i, p in enumerate(pasts):
        mine, off = int(tables[i, p // page]), p % page
        assert rel(k2[mine, :, off].float().cpu().reshape(-1), whole[i, heads * hd:(heads + kv) * hd]) <= 2.0 ** -8
        assert rel(v2[mine, :, :, off].float().cpu().reshape(-1), whole[i, (heads + kv) * hd:]) <= 2.0 ** -8
        q = qkv[i:i + 1, :heads * hd].float().cpu()
        k = torch.cat([case["ks"][i][:p], k2[mine, :, off].float().cpu().reshape(1, -1)])
        v = torch.cat([case["vs"][i][:p], v2[mine, :, :, off].float().cpu().reshape(1, -1)])
        ref = plain_rows(q, k, v, p, heads, kv, hd, window, 0.2, plain.distance_slopes(heads), plain.query_temperature([p], 0.7, 20))
        for out in (out1, out2):
            assert (out[i].float().cpu().double() - ref[0]).abs().max() <= 2.0 ** -6 * v.abs().max(), p


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens", [5, 1032])
def test_bias_and_cache_write_by_rows(ops, dtype, tokens):
    heads, kv, hd, page = 3, 2, 24, 8
    width, n_pages = (heads + 2 * kv) * hd, tokens // 8 + 3
    qkv, b = rnd((tokens, width), 1).to(dtype), rnd((width,), 2)
    slots = (torch.arange(tokens, dtype=torch.int32) + 8)
    slots[3] = -1
    k_pool, v_pool = torch.full((n_pages, kv, page, hd), 7.0, dtype=dtype).cuda(), torch.full((n_pages, kv, hd, page), 7.0, dtype=dtype).cuda()
    got = ops.rope_kv_write(qkv.cuda().clone(), torch.zeros(tokens, dtype=torch.int32).cuda(), heads, kv, hd, None, slots=slots.cuda(),
                            k_pool=k_pool, v_pool=v_pool, page_size=page, bias=b.cuda(), by_rows=True)
    ref = qkv.double() + b.double()
    assert rel(got[:, :heads * hd].float().cpu(), ref[:, :heads * hd]) <= tol(dtype, 1e-6, 2.0 ** -8)
    kept = torch.full((n_pages * page, kv, hd), 7.0, dtype=torch.float64), torch.full((n_pages * page, kv, hd), 7.0, dtype=torch.float64)
    stored = slots >= 0
    kept[0][slots[stored].long()] = ref[stored][:, heads * hd:(heads + kv) * hd].reshape(-1, kv, hd)
    kept[1][slots[stored].long()] = ref[stored][:, (heads + kv) * hd:].reshape(-1, kv, hd)
    assert rel(k_pool.float().cpu().permute(0, 2, 1, 3).reshape(-1, kv, hd), kept[0]) <= tol(dtype, 1e-6, 2.0 ** -8)
    assert rel(v_pool.float().cpu().permute(0, 3, 1, 2).reshape(-1, kv, hd), kept[1]) <= tol(dtype, 1e-6, 2.0 ** -8)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, dim, vdim, tau", [(2, 24, 40, 5.0), (3, 130, 20, 1.0)])
def test_gated_linear_attention_part(ops, dtype, heads, dim, vdim, tau):
    """The mixer through its own projections over portions (a long one, two tokens, one) from a slot with stale content,
    against the walk from zero; decays from nearly nothing to nearly one."""
    from from_scratch_inference_engine_amd.parts.base import make_part, prepare_parts

    w, rank, n = 72, 6, 61
    kw, vw = heads * dim, heads * vdim
    mats = {"q": (kw, w), "k": (kw, w), "v": (vw, w), "g": (vw, w), "a1": (rank, w), "a2": (kw, rank), "o": (w, vw)}
    t = {name: rnd(shape, 10 + i, shape[1] ** -0.5).to(dtype) for i, (name, shape) in enumerate(mats.items())}
    t["a2.b"], t["norm"] = rnd((kw,), 30, 4.0), 1 + rnd((vdim,), 31, 0.3)
    mixer = make_part("mixer", "gated_linear_attention", hidden_size=w, n_heads=heads, key_dim=dim, value_dim=vdim, decay_rank=rank,
                      tau=tau, norm_eps=1e-5)
    mixer.qkvg_weight = torch.cat([t[k] for k in "qkvg"]).cuda()
    mixer.a1_weight, mixer.a2_weight, mixer.o_weight = t["a1"].cuda(), t["a2"].cuda(), t["o"].cuda()
    mixer.a2_bias, mixer.norm_weight = t["a2.b"].cuda(), t["norm"].cuda()
    prepare_parts(mixer, torch.device("cuda:0"), dtype, {})
    x = rnd((n, w), 5).to(dtype)
    ref = plain.gla(x.double(), {k: v.double() for k, v in t.items()}, "", {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, 1e-5)
    state = torch.full((3, heads, dim, vdim), 9.0).cuda()
    state[1] = 0.0
    got, at = [], 0
    for size in (40, 2, 1, 17, 1):
        ctx = SimpleNamespace(q_starts=torch.tensor([0, size], dtype=torch.int32).cuda(), seq_slots=torch.tensor([1], dtype=torch.int32).cuda(),
                              partial_sums_ok=False)
        got.append(mixer.forward(x[at:at + size].cuda(), ctx, SimpleNamespace(state=state)).float().cpu())
        at += size
    assert rel(torch.cat(got), ref) <= tol(dtype, 5e-5, 0.04)
    assert (state[[0, 2]] == 9.0).all()


# ------------------------------------------------------------------------------------------------
# whole models
# ------------------------------------------------------------------------------------------------
def attention(heads, kv, dim, vdim, window, coef, every, scale=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 0.8 * dim ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if every:
        m["q_temp"] = {"coef": coef, "every": every}
    return m


def layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def model(width, vocab, positions, layers, eps=1e-5, cap=None):
    cfg = {"architecture": "Romepel", "width": width, "vocab": vocab, "max_positions": positions, "norm": {"eps": eps}, "layers": layers}
    return dict(cfg, logit_softcap=cap) if cap else cfg


# Configurations that differ from each other in every size and in the order of their layers.
# A: starts with attention without a feed-forward; values wider and narrower than keys, other windows and periods in
#    every layer, sizes that are no multiples of 8.
# B: keys and values of one size that the matrix-core kernels take, windows longer than a page and not a multiple of it,
#    one head, as many kv heads as heads, key channels beyond 128, no cap.
# C: heads of a size only the float32-arithmetic kernel takes in either precision; the whole past seen (no window).
# D: linear attention only (no paged cache); E: attention only (no state slots), a window of one position, odd widths.
# W: wide enough for the products that leave partial sums and for the decode step in one kernel.
CONFIG_A = model(88, 211, 300, [
    layer("attention", attention(6, 3, 20, 28, 13, 0.9, 10), None),
    layer("gla", {"heads": 3, "dim": 20, "vdim": 28, "tau": 5.0}, 100),
    layer("attention", attention(4, 2, 24, 12, 40, 0.5, 7), 60),
    layer("gla", {"heads": 2, "dim": 36, "vdim": 70, "tau": 11.0}, None),
    layer("attention", attention(10, 2, 12, 12, 21, 0.3, 25), 76),
], eps=1e-6, cap=6.0)
CONFIG_B = model(128, 300, 700, [
    layer("gla", {"heads": 1, "dim": 132, "vdim": 64, "tau": 2.0}, 256),
    layer("attention", attention(4, 2, 32, 32, 35, 0.4, 16), 128),
    layer("attention", attention(1, 1, 48, 48, 24, 0.7, 33), None),
    layer("attention", attention(3, 3, 64, 64, 101, 0.2, 50), 96),
    layer("gla", {"heads": 4, "dim": 16, "vdim": 16, "tau": 16.0}, None),
])
CONFIG_C = model(64, 150, 128, [
    layer("attention", attention(2, 1, 40, 40, None, 0.5, 9), 96),
    layer("gla", {"heads": 2, "dim": 16, "vdim": 32, "tau": 4.0}, 96),
    layer("attention", attention(3, 1, 10, 10, 17, 0.0, None), 36),
], cap=20.0)
CONFIG_D = model(48, 97, 80, [
    layer("gla", {"heads": 2, "dim": 24, "vdim": 40, "tau": 3.0}, 64),
    layer("gla", {"heads": 1, "dim": 40, "vdim": 24, "tau": 1.0}, None),
], cap=9.0)
CONFIG_E = model(54, 120, 75, [
    layer("attention", attention(2, 2, 16, 24, 1, 0.5, 4), 79),
    layer("attention", attention(7, 1, 32, 16, 19, 0.6, 11), None),
])
CONFIG_W = model(1024, 257, 400, [
    layer("attention", attention(8, 2, 64, 64, 70, 0.5, 30), 1160),
    layer("gla", {"heads": 4, "dim": 64, "vdim": 128, "tau": 6.0}, 1024),
    layer("attention", attention(12, 4, 32, 32, 50, 0.3, 40), 520),
], cap=15.0)
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D, "E": CONFIG_E, "W": CONFIG_W}
DECAY_RANK = {"A": 12, "B": 8, "C": 4, "D": 6, "E": 1, "W": 20}


def romepel_tensors(cfg, rank, seed):
    g = torch.Generator().manual_seed(seed)
    w, out = cfg["width"], {}

    def mat(name, rows, cols, bias=False, loud=1.0):
        out[name] = torch.randn(rows, cols, generator=g) * cols ** -0.5 * loud
        if bias:
            out[name + ".b"] = torch.randn(rows, generator=g) * 0.7 * loud

    def vec(name, n, spread, centre=0.0):
        out[name] = centre + torch.randn(n, generator=g) * spread
    mat("embed", cfg["vocab"], w)
    mat("pos", cfg["max_positions"], w)
    out["embed"] *= w ** 0.5
    out["pos"] *= 0.7 * w ** 0.5
    mat("head", cfg["vocab"], w)
    vec("final.norm", w, 0.3)
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        vec(p + "norm1", w, 0.3), vec(p + "norm1b", w, 0.3)
        if lay["type"] == "gla":
            kw, vw = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            mat(p + "mix.q", kw, w), mat(p + "mix.k", kw, w), mat(p + "mix.v", vw, w), mat(p + "mix.g", vw, w)
            mat(p + "mix.a1", rank, w), mat(p + "mix.a2", kw, rank), vec(p + "mix.a2.b", kw, 2.0, 2.0)
            vec(p + "mix.norm", m["vdim"], 0.3, 1.0), mat(p + "mix.o", w, vw)
        else:
            h, kv = m["heads"], m["kv_heads"]
            mat(p + "mix.q", h * m["dim"], w, True, 1.6), mat(p + "mix.k", kv * m["dim"], w, True, 1.6)
            mat(p + "mix.v", kv * m["vdim"], w, True), mat(p + "mix.o", w, h * m["vdim"])
        if lay["mlp"] is not None:
            vec(p + "norm2", w, 0.3), vec(p + "norm2b", w, 0.3)
            mat(p + "mlp.up", lay["mlp"]["ff"], w, True), mat(p + "mlp.down", w, lay["mlp"]["ff"], True)
            out[p + "mlp.act"] = torch.tensor([0.8, -0.5]) + 0.2 * torch.randn(2, generator=g)
    return {k: v.bfloat16().contiguous() for k, v in out.items()}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("romepel")
    out = {}
    for name, cfg in CONFIGS.items():
        d = helpers.make_model_dir(root / name, cfg, 0, tensors=romepel_tensors(cfg, DECAY_RANK[name], seed=1 + ord(name)))
        out[name] = (d, plain.read_config(d), plain.read_weights(d))
    return out


def close_enough(got, ref, dtype, what):
    """float32: 1e-4 of the largest logit; bfloat16: the difference's root mean square against the logits'."""
    got, ref = np.asarray(got, dtype=np.float64), np.asarray(ref, dtype=np.float64)
    assert got.shape == ref.shape and np.isfinite(got).all(), what
    if dtype == "float32":
        assert np.abs(got - ref).max() <= 1e-4 * np.abs(ref).max(), f"{what}: {np.abs(got - ref).max():.3e}"
    else:
        err = np.sqrt(((got - ref) ** 2).mean(-1)) / np.sqrt((ref ** 2).mean())
        assert err.max() <= 0.12 and err.mean() <= 0.04, f"{what}: worst row {err.argmax()} off by {err.max():.3f} of the logits' size, mean {err.mean():.3f}"


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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_model_whole_in_portions_decoded_and_batched(models, name, dtype):
    """The same requests whole, token by token (through the captured decode graphs), in portions down to two tokens and
    one, and in batches of unequal requests that start and end at different steps in a pool so small that pages and
    state slots are taken again: all against the plain implementation."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models[name]
    vocab = cfg["vocab"]
    seqs = {"a": helpers.token_ids(vocab, 75, 1), "b": helpers.token_ids(vocab, 1, 2), "c": helpers.token_ids(vocab, 33, 3),
            "d": helpers.token_ids(vocab, 127, 4), "e": helpers.token_ids(vocab, 18, 5)}
    ref = {r: plain.forward(cfg, w, ids).numpy() for r, ids in seqs.items()}
    runner = Runner(load_model(d, dtype=dtype), page_size=8, num_pages=34, max_requests=3)
    assert runner.graphs.enabled and runner.max_position == cfg["max_positions"]
    # whole, one after the other (each takes the pages and the slot the last one gave back)
    got = step_through(runner, [[(r, len(ids))] for r, ids in seqs.items()], seqs)
    for r in seqs:
        close_enough(got[r], ref[r], dtype, f"{name} whole {r}")
    # a first portion, then token by token: decode steps replay graphs, the state and the cache go on
    for r, head in (("a", 40), ("c", 1)):
        got = step_through(runner, [[(r, head)]] + [[(r, 1)]] * (len(seqs[r]) - head), {r: seqs[r]})
        close_enough(got[r], ref[r], dtype, f"{name} decode {r}")
    assert runner.graphs.replays > 50
    # portions of changing size
    sizes, plan, left = [2, 7, 1, 16, 3, 2, 33, 8, 64], [], len(seqs["d"])
    while left:
        n = min(sizes[len(plan) % len(sizes)], left)
        plan.append([("d", n)])
        left -= n
    close_enough(step_through(runner, plan, {"d": seqs["d"]})["d"], ref["d"], dtype, f"{name} portions")
    # batches: three slots, five requests; portions beside single tokens; b and e start where a and c ended
    plan = [[("a", 30), ("c", 2), ("b", 1)], [("a", 1), ("c", 20), ("e", 3)], [("c", 11), ("a", 44), ("e", 1)],
            [("e", 14), ("d", 9)], [("d", 117)], [("d", 1)]]
    got = step_through(runner, plan, seqs)
    for r in seqs:
        close_enough(got[r], ref[r], dtype, f"{name} batched {r}")
    assert all(a.pages_issued_again() for a in runner.manager.allocators)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["D", "E"])
def test_model_of_one_kind_of_layer(models, name, dtype):
    """A model with state slots and no paged cache, and one with a paged cache and no state (and a window of one
    position): whole, a portion and then token by token, and two requests together, in a pool that is used again."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models[name]
    seqs = {"a": helpers.token_ids(cfg["vocab"], 70, 1), "b": helpers.token_ids(cfg["vocab"], 23, 2)}
    ref = {r: plain.forward(cfg, w, ids).numpy() for r, ids in seqs.items()}
    runner = Runner(load_model(d, dtype=dtype), page_size=8, num_pages=14, max_requests=2)
    got = step_through(runner, [[(r, len(ids))] for r, ids in seqs.items()], seqs)
    for r in seqs:
        close_enough(got[r], ref[r], dtype, f"{name} whole {r}")
    got = step_through(runner, [[("a", 37)]] + [[("a", 1)]] * 33, {"a": seqs["a"]})
    close_enough(got["a"], ref["a"], dtype, f"{name} decode")
    got = step_through(runner, [[("a", 50), ("b", 2)], [("a", 19), ("b", 1)], [("a", 1), ("b", 17)], [("b", 3)]], seqs)
    for r in seqs:
        close_enough(got[r], ref[r], dtype, f"{name} batched {r}")


@pytest.mark.parametrize("copies", [False, True])
def test_wide_model_takes_the_fused_steps(models, copies, monkeypatch):
    """Sizes at which decode steps start attention from the q/k/v product's partial sums, portions of 17 to 64 tokens
    are added up by the kernel that writes the cache, and the feed-forward's bias waits for the norm: batches of single
    tokens and portions, with the large matrices' second copies and without, against the plain implementation."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner
    from from_scratch_inference_engine_amd.parts import attention as attention_part
    from from_scratch_inference_engine_amd.parts.linear import Linear

    d, cfg, w = models["W"]
    monkeypatch.setattr(Linear, "streamed_copy_from", 0 if copies else 1 << 40)
    calls = {"qkv": 0, "by_rows": 0}
    real_qkv, real_write = attention_part.ops.attention_mfma_qkv, attention_part.ops.rope_kv_write
    monkeypatch.setattr(attention_part.ops, "attention_mfma_qkv", lambda *a, **k: (calls.__setitem__("qkv", calls["qkv"] + 1), real_qkv(*a, **k))[1])
    monkeypatch.setattr(attention_part.ops, "rope_kv_write",
                        lambda *a, **k: (calls.__setitem__("by_rows", calls["by_rows"] + (k.get("parts") is not None)), real_write(*a, **k))[1])
    runner = Runner(load_model(d, dtype="bfloat16"), page_size=16, num_pages=48, max_requests=4)
    seqs = {r: helpers.token_ids(cfg["vocab"], n, 40 + n) for r, n in (("a", 110), ("b", 31), ("c", 95), ("d", 12))}
    ref = {r: plain.forward(cfg, w, ids).numpy() for r, ids in seqs.items()}
    plan = [[("a", 40)], [("a", 20), ("b", 10)], [("c", 80), ("a", 9)]] + [[("a", 1), ("b", 1), ("c", 1)]] * 15
    plan += [[("a", 2), ("d", 9)]] + [[("a", 1), ("b", 1), ("d", 1)]] * 3 + [[("a", 1), ("b", 1)]] * 3 + [[("a", 18)]]
    got = step_through(runner, plan, seqs)
    for r in seqs:
        close_enough(got[r], ref[r], "bfloat16", f"wide {r}")
    assert calls["qkv"] > 0 and calls["by_rows"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_passes_windows_and_periods(models, dtype):
    """300 tokens decoded one by one: every window moves over decoded tokens and gives its pages back, the queries'
    factor steps up at every period's end, the state is carried all the way."""
    from from_scratch_inference_engine_amd import load_model
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models["B"]
    ids = helpers.token_ids(cfg["vocab"], 330, 12)
    ref = plain.forward(cfg, w, ids).numpy()
    runner = Runner(load_model(d, dtype=dtype), page_size=16, num_pages=24, max_requests=1)
    got = step_through(runner, [[("a", 30)]] + [[("a", 1)]] * 300, {"a": ids})
    close_enough(got["a"], ref, dtype, "long decoding")


def test_positions_beyond_the_table_are_refused(models):
    from from_scratch_inference_engine_amd import LLM, load_model
    from from_scratch_inference_engine_amd.engine.context import StepEntry
    from from_scratch_inference_engine_amd.engine.model import Runner

    d, cfg, w = models["E"]  # 75 positions
    runner = Runner(load_model(d, dtype="float32"), page_size=8, num_pages=16, max_requests=1)
    ids = helpers.token_ids(cfg["vocab"], 76, 3)
    rc = runner.manager.open("a")
    with pytest.raises(ValueError, match="limit of 75"):
        runner.step([StepEntry(rc, ids, [])])
    out = runner.step([StepEntry(rc, ids[:75], [74])]).cpu().numpy()
    close_enough(out, plain.forward(cfg, w, ids[:75]).numpy()[74:], "float32", "the last position")
    with pytest.raises(ValueError, match="limit of 75"):
        runner.step([StepEntry(rc, ids[75:], [0])])
    with pytest.raises(Exception, match="75"):
        LLM(d, dtype="float32", block_size=8, num_blocks=32, max_batch=1, eos_id=-1).engine.add_request(ids[:70], max_tokens=7)


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_engine(models, name):
    """Prompts of unequal length generated together through the LLM entry point and its scheduler (three at a time,
    portions of at most 16 tokens), in float32: the tokens are the plain implementation's greedy ones; long enough that
    decode steps run from graphs and pages fill up."""
    from from_scratch_inference_engine_amd import GenerationConfig, LLM

    d, cfg, w = models[name]
    prompts = [helpers.token_ids(cfg["vocab"], n, 20 + n) for n in (1, 9, 40, 23)]
    n_new = 48
    llm = LLM(d, dtype="float32", block_size=8, num_blocks=64, max_batch=3, eos_id=-1, prefill_chunk=16)
    got = llm.generate_ids_batch(prompts, GenerationConfig(max_tokens=n_new))
    for prompt, mine in zip(prompts, got):
        assert len(mine) == n_new
        logits = plain.forward(cfg, w, prompt + mine)[len(prompt) - 1:-1]
        top2 = logits.topk(2, dim=-1).values
        for i, tok in enumerate(mine):  # the plain choice, unless the two best are a rounding apart
            assert tok == int(logits[i].argmax()) or (top2[i, 0] - logits[i, tok]) <= 1e-4 * logits.abs().max(), (len(prompt), i)
    assert llm.engine.runner.graphs.replays > 0


@pytest.mark.parametrize("name", ["A", "D", "E"])
def test_replay_program_runs_the_model(models, tmp_path, name):
    """bin/trace_run on the architecture (mixed layers, state only, cache only): a prompt in portions beside another
    request's single tokens."""
    d, cfg, w = models[name]
    a, b = helpers.token_ids(cfg["vocab"], 50, 7), helpers.token_ids(cfg["vocab"], 20, 8)
    tb = helpers.TraceBuilder()
    tb.step([("a", a[:17], [16]), ("b", b[:1], [0])])
    for i in range(1, 20):
        lo, hi = 17 + (i - 1) * 2, min(50, 17 + i * 2)
        entries = [("b", b[i:i + 1], [0])] + ([("a", a[lo:hi], list(range(hi - lo)))] if lo < 50 else [])
        tb.step(entries, end=["b"] if i == 19 else [])
    tb.step([], end=["a"])
    for dtype in ("float32", "bfloat16"):
        per = helpers.collect(tb, helpers.run_trace(d, dtype, tb.steps, 128, tmp_path / dtype))
        for rid, ids in (("a", a), ("b", b)):
            ref = plain.forward(cfg, w, ids).numpy()
            pos = sorted(per[rid])
            close_enough(np.stack([per[rid][p] for p in pos]), ref[pos], dtype, f"replay {rid}")


def test_command_line_writes_a_random_model_and_generates(tmp_path):
    """random-model from a config.json that states the decays' rank (``a_rank``; a folder's config.json may leave it to
    the checkpoint), then generate from that folder."""
    import os
    import subprocess
    import sys

    raw = copy.deepcopy(CONFIG_A)
    for lay in raw["layers"]:
        if lay["type"] == "gla":
            lay["mixer"]["a_rank"] = 6
    (tmp_path / "cfg.json").write_text(json.dumps(raw))
    env = dict(os.environ, PYTHONPATH=str(helpers.ROOT))
    base = [sys.executable, "-m", "from_scratch_inference_engine_amd"]
    made = subprocess.run(base + ["random-model", "--config", str(tmp_path / "cfg.json"), "--out", str(tmp_path / "m"), "--seed", "5"],
                          capture_output=True, text=True, env=env, timeout=300)
    assert made.returncode == 0, made.stderr[-2000:]
    ids = [3, 1, 4, 1, 5, 9, 2, 6]
    a = subprocess.run(base + ["generate", "--model-dir", str(tmp_path / "m"), "--prompt-ids", " ".join(map(str, ids)), "--max-tokens", "12",
                               "--num-blocks", "64", "--max-batch", "4", "--dtype", "float32"], capture_output=True, text=True, env=env, timeout=300)
    assert a.returncode == 0, a.stderr[-2000:]
    tokens = [int(t) for t in a.stdout.strip().splitlines()[-1].split()]
    assert len(tokens) == 12
    cfg, w = plain.read_config(tmp_path / "m"), plain.read_weights(tmp_path / "m")
    logits = plain.forward(cfg, w, ids + tokens)[len(ids) - 1:-1]
    for i, t in enumerate(tokens):
        assert t == int(logits[i].argmax()) or (logits[i].max() - logits[i, t]) <= 1e-4 * logits.abs().max(), i
