"""Nenizen's configuration, registry entry, schedule and tensor list, and its plain implementation against itself (CPU)."""

import copy
import math

import numpy as np
import pytest

import helpers
import plain_nenizen as plain
from from_scratch_inference_engine_amd import ops
from from_scratch_inference_engine_amd.config import ConfigError, NenizenConfig
from from_scratch_inference_engine_amd.models import build_model_spec, known_architectures, parse_config
from from_scratch_inference_engine_amd.parts import OriginMix
from from_scratch_inference_engine_amd.parts.base import make_part
from from_scratch_inference_engine_amd.weights.loader import expected_tensors

RAW = {"architecture": "Nenizen", "width": 40, "vocab": 77, "norm": {"eps": 1e-4}, "embedding": {"scale": 3.0},
       "logit_softcap": 12.5, "loop": {"start": 1, "stop": 3, "times": 3},
       "layers": [
           {"type": "latent_attention_2", "mlp": {"kind": "dense", "ff": 52, "limit": 2.5},
            "mixer": {"heads": 3, "dim": 10, "rot_dim": 6, "vdim": 14, "kv_rank": 22, "q_rank": 18, "scale": 0.21,
                      "mask": {"size": 9}, "rot": {"base": 700.0, "dims": 6}}},
           {"type": "latent_attention", "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 5, "top": 2},
                                                "shared": {"ff": 36}},
            "mixer": {"heads": 2, "dim": 12, "rot_dim": 4, "vdim": 8, "kv_rank": 30, "scale": 0.3, "rot": {"base": 90.0, "dims": 4}}},
           {"type": "latent_attention_3", "mlp": None,
            "mixer": {"heads": 5, "dim": 6, "rot_dim": 2, "vdim": 7, "kv_rank": 12, "q_rank": 9, "scale": 0.4,
                      "rot": {"base": 1e4, "dims": 2}}},
           {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 20, "limit": 0.75},
            "mixer": {"heads": 1, "dim": 8, "rot_dim": 8, "vdim": 9, "kv_rank": 16, "scale": 0.25, "rot": {"base": 50.0, "dims": 8}}}]}


def test_registered_and_parsed():
    assert "Nenizen" in known_architectures()
    cfg = parse_config(RAW)
    assert isinstance(cfg, NenizenConfig) and (cfg.width, cfg.vocab, cfg.norm_eps, cfg.embedding_scale) == (40, 77, 1e-4, 3.0)
    assert (cfg.loop.start, cfg.loop.stop, cfg.loop.times, cfg.logit_softcap) == (1, 3, 3, 12.5)
    assert [layer.mixer.window for layer in cfg.layers] == [9, None, None, None]
    assert [layer.mixer.q_rank for layer in cfg.layers] == [18, None, 9, None]
    assert cfg.layers[1].mlp.shared_ff == 36 and cfg.layers[2].mlp is None and cfg.layers[3].mlp.limit == 0.75
    assert parse_config(cfg.to_dict()) == cfg
    bare = copy.deepcopy(RAW)
    del bare["logit_softcap"], bare["loop"], bare["layers"][1]["mlp"]["shared"]
    cfg = parse_config(bare)
    assert cfg.logit_softcap is None and cfg.loop is None and cfg.layers[1].mlp.shared_ff is None
    assert parse_config(cfg.to_dict()) == cfg


def test_schedule_runs_the_loop_with_an_entrance_before_every_pass():
    spec = build_model_spec(parse_config(RAW))
    assert [c.layer for c in spec.schedule] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [c.layer for c in spec.schedule] == [i for i, _ in plain.runs(RAW)]
    assert [c.entrance_number if c.entrance else None for c in spec.schedule] == [n for _, n in plain.runs(RAW)]
    assert all(c.cache_of is None for c in spec.schedule)  # every pass keeps a cache of its own
    (entrance,) = spec.entrances()
    assert isinstance(entrance, OriginMix) and entrance in spec.all_parts() and entrance.numbers == 3
    assert all(norm.adds_partial_sums for norm in spec.stream_norms())
    for loop, order in (({"start": 0, "stop": 4, "times": 1}, [0, 1, 2, 3]), ({"start": 3, "stop": 4, "times": 2}, [0, 1, 2, 3, 3])):
        spec = build_model_spec(parse_config({**RAW, "loop": loop}))
        assert [c.layer for c in spec.schedule] == order == [i for i, _ in plain.runs({**RAW, "loop": loop})]
    spec = build_model_spec(parse_config({**RAW, "loop": None}))
    assert [c.layer for c in spec.schedule] == [0, 1, 2, 3] and not spec.entrances()
    assert "loop.in" not in expected_tensors(spec.bindings)


def test_tensor_list_and_parts():
    spec = build_model_spec(parse_config(RAW))
    names = expected_tensors(spec.bindings)
    want = {"embed": (77, 40), "final.norm": (40,), "loop.in": (40, 80), "loop.step": (3, 40), "l0.norm1b": (40,),
            "l0.mix.dq": (18, 40), "l0.mix.dq.norm": (18,), "l0.mix.uq": (48, 18), "l0.mix.dkv": (28, 40),
            "l0.mix.dkv.norm": (22,), "l0.mix.uk": (30, 22), "l0.mix.uv": (42, 22), "l0.mix.g": (3, 40), "l0.mix.o": (40, 42),
            "l0.mlp.gate": (52, 40), "l0.mlp.down": (40, 52), "l1.mix.q": (32, 40), "l1.mix.g": (16, 40),
            "l1.mlp.router": (5, 40), "l1.mlp.e4.up": (24, 40), "l1.mlp.e0.down": (40, 24), "l1.mlp.shared.gate": (36, 40),
            "l1.mlp.shared.down": (40, 36), "l2.mix.sink": (5,), "l2.norm1": (40,)}
    for name, shape in want.items():
        assert tuple(names[name].shape) == shape, name
    for name in ("head", "l0.mix.sink", "l0.mix.q", "l1.mix.dq", "l1.mix.sink", "l2.mix.g", "l2.norm2", "l2.mlp.gate", "l1.mlp.e5.up"):
        assert name not in names, name
    assert set(spec.ignore_unexpected) == {"l2.norm2", "l2.norm2b"}
    a, b, c, d = (layer.mixer for layer in spec.layers)
    assert (a.gate, b.gate, c.gate, d.gate) == ("heads", "values", None, "values")
    assert (a.has_sink, b.has_sink, c.has_sink) == (False, False, True) and (a.window, c.window) == (9, None)
    assert a.kernel_pairs == -3 and b.kernel_pairs == 2 and c.kernel_pairs == -1
    dense, experts = spec.layers[0].ffn, spec.layers[1].ffn
    assert dense._gate_act.args == (3, 2.5, 1.702) and spec.layers[3].ffn._gate_act.limit == 0.75
    assert experts.shared.intermediate_size == 36 and experts.scores == "softmax" and not experts.renorm and not experts.has_correction
    assert experts.groups == 1 and experts.top == 2 and experts.shared.activation == "silu"
    assert spec.lm_head.softcap == 12.5 and spec.embedding.scale == 3.0


@pytest.mark.parametrize("edit, message", [
    (lambda r: r["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda r: r["layers"][0]["mixer"].pop("mask"), "mask"),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=4), "rot.dims"),
    (lambda r: r["layers"][1]["mixer"].update(rot_dim=3, rot={"base": 10.0, "dims": 3}), "even"),
    (lambda r: r["layers"][1]["mixer"].pop("rot"), "rot"),
    (lambda r: r["layers"][1]["mixer"].update(scale=0), "scale"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(top=6), "top 6"),
    (lambda r: r["layers"][1]["mlp"].pop("router"), "router"),
    (lambda r: r["layers"][1]["mlp"].update(kind="sparse"), "sparse"),
    (lambda r: r["layers"][1]["mlp"]["shared"].pop("ff"), "shared"),
    (lambda r: r["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda r: r["layers"][2].update(type="latent_attention_4"), "not a mixer"),
    (lambda r: r["layers"][2].update(mlp=[1]), "mlp"),
    (lambda r: r["loop"].update(stop=5), "loop"),
    (lambda r: r["loop"].update(start=3), "loop"),
    (lambda r: r["loop"].update(times=0), "times"),
    (lambda r: r.update(layers=[]), "layers"),
    (lambda r: r.pop("vocab"), "vocab"),
])
def test_refused(edit, message):
    raw = copy.deepcopy(RAW)
    edit(raw)
    with pytest.raises(ConfigError, match=message):
        parse_config(raw)


def test_parts_that_do_not_go_together_are_refused():
    with pytest.raises(ops.KernelError, match="positive"):
        ops.GateAct("clipped", limit=0.0, slope=1.0)
    with pytest.raises(ops.KernelError, match="unknown gate"):
        make_part("feed_forward", "gated", hidden_size=8, intermediate_size=16, activation="swoosh")
    with pytest.raises(ValueError, match="gate"):
        make_part("mixer", "latent_attention", hidden_size=16, n_heads=2, head_dim=8, rot_dim=0, value_dim=8, kv_rank=8, q_rank=None,
                  scale=1.0, norm_eps=1e-5, position=make_part("position", "none"), gate="tokens")
    with pytest.raises(ValueError, match="whole output"):
        make_part("feed_forward", "routed_experts", hidden_size=8, intermediate_size=8, n_experts=2, top=1,
                  shared=make_part("feed_forward", "plain", hidden_size=8, intermediate_size=16, defer_bias=True))
    with pytest.raises(ValueError, match="passes"):
        make_part("entrance", "origin_mix", hidden_size=8, numbers=0)


# ------------------------------------------------------------------------------------------------
# the plain implementation
# ------------------------------------------------------------------------------------------------
def test_plain_gate_rotation_window_and_sink():
    g, u, lim = np.array([5.0, -9.0, 1.0]), np.array([9.0, -9.0, 0.5]), 2.0
    want = [2 / (1 + math.exp(-1.702 * 2)) * 3.0, -9 / (1 + math.exp(1.702 * 9)) * -1.0, 1 / (1 + math.exp(-1.702)) * 1.5]
    assert np.allclose(plain.clipped_gate(g, u, lim), want, rtol=1e-14)
    x = np.arange(1.0, 9.0).reshape(2, 1, 4)
    a, b = plain.rotate(x, [0, 3], 100.0, True), plain.rotate(x, [0, 3], 100.0, False)
    assert np.array_equal(a[0], x[0]) and np.array_equal(b[0], x[0])
    angles = [3.0, 3.0 / 10.0]
    for out, pairs in ((a[1, 0], ((0, 1), (2, 3))), (b[1, 0], ((0, 2), (1, 3)))):
        for angle, (i, j) in zip(angles, pairs):
            v = complex(x[1, 0, i], x[1, 0, j]) * complex(math.cos(angle), math.sin(angle))
            assert np.allclose([out[i], out[j]], [v.real, v.imag], rtol=1e-13)
    assert plain.visible(6, 3)[5].tolist() == [False, False, False, True, True, True] and plain.visible(6)[2].tolist() == [True] * 3 + [False] * 3
    v = np.ones((2, 1, 1))
    out = plain.softmax_mix(np.zeros((1, 2, 2)), plain.visible(2), v, np.array([math.log(3.0)]))
    assert np.allclose(out[:, 0, 0], [1 / 4, 2 / 5])


def test_plain_router_keeps_the_scores_of_the_whole_softmax():
    z = np.log(np.array([[1.0, 5.0, 2.0, 2.0]]))
    ids, weights = plain.route(z, 2)
    assert ids.tolist() == [[1, 2]] and np.allclose(weights, [[0.5, 0.2]])


@pytest.mark.parametrize("fault", ["window", "sink", "gate a value", "gate a head", "interleaved", "half", "limit", "up offset",
                                   "shared", "renormalised", "choice", "entrance", "step", "passes", "embedding", "query norm",
                                   "latent norm", "key part", "embedding scale"])
def test_a_fault_in_the_plain_model_shows(monkeypatch, fault):
    """The weights of the model tests make a small fault of each mechanism visible in the logits, by hundreds of times the
    tolerance of the float32 comparisons."""
    from test_nenizen_gpu import CONFIG_A, nenizen_tensors

    w = {k: v.double().numpy() for k, v in nenizen_tensors(CONFIG_A, 66).items()}
    ids = helpers.token_ids(CONFIG_A["vocab"], 70, 4)
    good = plain.forward(CONFIG_A, w, ids)
    cfg = copy.deepcopy(CONFIG_A)
    kinds, keep = copy.deepcopy(plain.KINDS), {n: getattr(plain, n) for n in ("clipped_gate", "route", "enter_pass", "latent_keys", "rms_norm")}
    if fault == "window":
        for layer in cfg["layers"]:
            if "mask" in layer["mixer"]:
                layer["mixer"]["mask"]["size"] += 1
    elif fault == "sink":
        kinds["latent_attention_3"]["sink"] = False
    elif fault == "gate a value":
        kinds["latent_attention"]["gate"] = None
    elif fault == "gate a head":
        kinds["latent_attention_2"]["gate"] = None
    elif fault == "interleaved":
        kinds["latent_attention"]["interleaved"] = False
    elif fault == "half":
        kinds["latent_attention_3"]["interleaved"] = True
    elif fault == "limit":
        for layer in cfg["layers"]:
            if layer["mlp"] and layer["mlp"]["kind"] == "dense":
                layer["mlp"]["limit"] *= 1.5
    elif fault == "up offset":
        monkeypatch.setattr(plain, "clipped_gate", lambda g, u, lim: keep["clipped_gate"](g, u - 1.0, lim))
    elif fault == "shared":
        for layer in cfg["layers"]:
            if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                layer["mlp"]["shared"] = None
    elif fault == "renormalised":
        monkeypatch.setattr(plain, "route", lambda z, top, m=None: (lambda i, s: (i, s / s.sum(-1, keepdims=True)))(*keep["route"](z, top, m)))
    elif fault == "choice":
        monkeypatch.setattr(plain, "route", lambda z, top, m=None: keep["route"](z, top - 1, m))
    elif fault == "entrance":
        monkeypatch.setattr(plain, "enter_pass", lambda x, x0, w, n: keep["enter_pass"](x0, x, w, n))
    elif fault == "step":
        monkeypatch.setattr(plain, "enter_pass", lambda x, x0, w, n: keep["enter_pass"](x, x0, w, 0))
    elif fault == "passes":
        cfg["loop"]["times"] -= 1
    elif fault == "embedding":
        monkeypatch.setattr(plain, "enter_pass", lambda x, x0, w, n: keep["enter_pass"](x, x, w, n))
    elif fault == "query norm":
        w = {k: (np.ones_like(v) if k.endswith("dq.norm") else v) for k, v in w.items()}
    elif fault == "latent norm":
        w = {k: (np.ones_like(v) if k.endswith("dkv.norm") else v) for k, v in w.items()}
    elif fault == "key part":
        monkeypatch.setattr(plain, "latent_keys", lambda *a: (lambda c, r: (c, 0.0 * r))(*keep["latent_keys"](*a)))
    else:
        cfg["embedding"]["scale"] *= 1.5
    monkeypatch.setattr(plain, "KINDS", kinds)
    bad = plain.forward(cfg, w, ids)
    off = np.sqrt(((bad - good) ** 2).mean(-1) / (good ** 2).mean())
    assert off.max() > 0.02, f"{fault}: {off.max():.3f}"
