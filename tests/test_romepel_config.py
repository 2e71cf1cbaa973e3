"""Romepel's configuration, registry entry and tensor list, and its plain implementation against itself (CPU)."""

import copy
import math

import pytest
import torch

import helpers
import plain_romepel as plain
from from_scratch_inference_engine_amd.config import ConfigError, RomepelConfig
from from_scratch_inference_engine_amd.models import build_model_spec, known_architectures, parse_config
from from_scratch_inference_engine_amd.models.romepel import distance_slopes
from from_scratch_inference_engine_amd.parts.base import make_part
from from_scratch_inference_engine_amd.weights.loader import expected_tensors

RAW = {"architecture": "Romepel", "width": 40, "vocab": 77, "max_positions": 90, "norm": {"eps": 1e-4}, "logit_softcap": 12.5,
       "layers": [
           {"type": "attention", "mlp": None,
            "mixer": {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 14, "scale": 0.21, "mask": {"size": 9},
                      "q_temp": {"coef": 0.4, "every": 12}}},
           {"type": "gla", "mixer": {"heads": 2, "dim": 12, "vdim": 10, "tau": 4.0}, "mlp": {"kind": "dense", "ff": 64}},
           {"type": "attention", "mlp": {"kind": "dense", "ff": 52},
            "mixer": {"heads": 5, "kv_heads": 5, "dim": 8, "vdim": 8, "scale": 0.4, "mask": {"size": 30},
                      "q_temp": {"coef": 0.1, "every": 5}}},
           {"type": "gla", "mixer": {"heads": 3, "dim": 4, "vdim": 6, "tau": 2.5}, "mlp": None}]}


def test_registered_and_parsed():
    assert "Romepel" in known_architectures()
    cfg = parse_config(RAW)
    assert isinstance(cfg, RomepelConfig) and cfg.width == 40 and cfg.vocab == 77 and cfg.logit_softcap == 12.5
    assert cfg.max_positions == 90 and cfg.norm_eps == 1e-4
    assert [layer.kind for layer in cfg.layers] == ["attention", "gla", "attention", "gla"]
    assert [layer.ff for layer in cfg.layers] == [None, 64, 52, None]
    assert cfg.layers[0].mixer.window == 9 and cfg.layers[0].mixer.temperature == (0.4, 12.0)
    assert parse_config(cfg.to_dict()) == cfg
    bare = copy.deepcopy(RAW)
    del bare["logit_softcap"], bare["layers"][0]["mixer"]["mask"], bare["layers"][2]["mixer"]["q_temp"]
    cfg = parse_config(bare)
    assert cfg.logit_softcap is None and cfg.layers[0].mixer.window is None and cfg.layers[2].mixer.temperature is None
    assert parse_config(cfg.to_dict()) == cfg


def test_decay_rank_comes_from_the_checkpoint_and_the_tensor_list_follows():
    cfg = parse_config(RAW)
    with pytest.raises(ConfigError, match="a1"):
        build_model_spec(cfg)
    done = cfg.completed_from({"l1.mix.a1": (5, 40), "l3.mix.a1": (7, 40)})
    assert done.layers[1].mixer.decay_rank == 5 and done.layers[3].mixer.decay_rank == 7 and parse_config(done.to_dict()) == done
    spec = build_model_spec(done)
    names = expected_tensors(spec.bindings)
    want = {"embed": (77, 40), "pos": (90, 40), "head": (77, 40), "final.norm": (40,), "l0.norm1": (40,), "l0.norm1b": (40,),
            "l0.mix.q": (60, 40), "l0.mix.q.b": (60,), "l0.mix.k": (30, 40), "l0.mix.k.b": (30,), "l0.mix.v": (42, 40),
            "l0.mix.v.b": (42,), "l0.mix.o": (40, 84), "l1.mix.a2": (24, 5), "l1.mix.a2.b": (24,), "l1.mix.norm": (10,),
            "l1.mlp.up": (64, 40), "l1.mlp.up.b": (64,), "l1.mlp.act": (2,), "l1.mlp.down": (40, 64), "l1.mlp.down.b": (40,),
            "l2.norm2b": (40,), "l3.mix.a1": (7, 40)}
    for name, shape in want.items():
        assert tuple(names[name].shape) == shape, name
    for name in ("l0.norm2", "l0.mlp.up", "l3.norm2b", "l0.mix.o.b", "l1.mix.q.b"):
        assert name not in names
    assert spec.lm_head.softcap == 12.5 and spec.layers[0].ffn is None and spec.embedding.n_positions == 90
    # the feed-forward leaves its last bias to the norm behind it
    assert spec.layers[1].ffn.defer_bias and spec.layers[1].ffn_post_norm.adds_delta_bias


def test_slopes_fall_by_a_power_a_head():
    for heads in (1, 3, 8, 12):
        got = distance_slopes(heads)
        assert got[-1] == 2.0 ** -8 and all(math.isclose(b / a, 2.0 ** (-8 / heads), rel_tol=1e-12) for a, b in zip(got, got[1:]))
        assert torch.allclose(torch.tensor(got, dtype=torch.float64), plain.distance_slopes(heads), rtol=1e-15)


@pytest.mark.parametrize("edit, message", [
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda r: r["layers"][0]["mixer"].pop("vdim"), "vdim"),
    (lambda r: r["layers"][0]["mixer"].update(scale=0.0), "scale"),
    (lambda r: r["layers"][0]["mixer"].update(mask={}), "mask.size"),
    (lambda r: r["layers"][0]["mixer"].update(mask={"size": 0}), "mask.size"),
    (lambda r: r["layers"][0]["mixer"].update(q_temp={"coef": 0.1}), "q_temp.every"),
    (lambda r: r["layers"][1]["mixer"].pop("tau"), "tau"),
    (lambda r: r["layers"][1].update(type="conv"), "not a mixer"),
    (lambda r: r["layers"][1].update(mlp={"kind": "moe", "ff": 8}), "dense"),
    (lambda r: r["layers"][1].update(mlp={"kind": "dense"}), "mlp.ff"),
    (lambda r: r.pop("max_positions"), "max_positions"),
    (lambda r: r.update(layers=[]), "layers"),
])
def test_refused(edit, message):
    raw = copy.deepcopy(RAW)
    edit(raw)
    with pytest.raises(ConfigError, match=message):
        parse_config(raw)


def test_parts_that_do_not_go_together_are_refused():
    ffn = make_part("feed_forward", "plain", hidden_size=8, intermediate_size=16, defer_bias=True)
    norm = make_part("norm", "rms_norm", hidden_size=8, eps=1e-5)
    with pytest.raises(ValueError, match="last bias"):
        make_part("block", "pre_norm", mixer_norm=norm, mixer=None, ffn_norm=norm, ffn=ffn)
    args = dict(hidden_size=32, n_heads=4, n_kv_heads=2, head_dim=8, qkv_bias=True, position=make_part("position", "none"))
    with pytest.raises(ValueError, match="slopes"):
        make_part("mixer", "gqa_attention", slopes=[0.5, 0.25], **args)
    with pytest.raises(ValueError, match="slopes"):
        make_part("mixer", "gqa_attention", slopes=[0.5] * 4, window=16, pool=4, **args)
    with pytest.raises(ValueError, match="period"):
        make_part("mixer", "gqa_attention", query_temperature=(0.5, 0.0), **args)


# ------------------------------------------------------------------------------------------------
# the plain implementation
# ------------------------------------------------------------------------------------------------
def test_plain_activation():
    act = torch.tensor([0.3, -0.8], dtype=torch.float64)
    up, down = math.log(1 + math.exp(0.3)), 0.5 + math.log(1 + math.exp(-0.8))
    for z, want in ((2.0, up * 4 + 1), (-2.0, down * (math.exp(-2) + 1) - 1), (0.0, 0.0), (-1e-9, -5e-10)):
        assert plain.xielu(torch.tensor([z], dtype=torch.float64), act).item() == pytest.approx(want, rel=1e-12, abs=1e-18)


def test_plain_window_bias_and_temperature():
    assert plain.window_mask([5], range(8), 3)[0].tolist() == [False, False, False, True, True, True, False, False]
    assert plain.window_mask([1], range(3), 3)[0].tolist() == [True, True, False]
    t = plain.query_temperature([0, 6, 7, 14, 15, 1000], 0.5, 8)
    want = [1.0, 1.0, 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(3), 1 + 0.5 * math.log(126)]
    assert torch.allclose(t, torch.tensor(want, dtype=torch.float64), rtol=1e-14)
    # equal keys: the weights of a head are powers of exp(-slope)
    q, k = torch.zeros(1, 2, 4, dtype=torch.float64), torch.ones(5, 1, 4, dtype=torch.float64)
    v = torch.eye(5, dtype=torch.float64).unsqueeze(1)
    w = plain.biased_attention(q, k, v, 4, 1.0, 4, plain.distance_slopes(2), torch.ones(1, dtype=torch.float64))[0]
    for h, slope in enumerate((2.0 ** -4, 2.0 ** -8)):
        e = [math.exp(-slope * d) for d in (3, 2, 1, 0)]
        assert torch.allclose(w[h], torch.tensor([0.0] + [x / sum(e) for x in e], dtype=torch.float64), rtol=1e-12)


@pytest.mark.parametrize("fault", ["window", "slope", "temperature", "position", "state", "bias", "activation", "kv head"])
def test_a_fault_in_the_plain_model_shows(monkeypatch, fault):
    """The weights of the model tests make a small fault of each mechanism visible in the logits, by hundreds of times the
    tolerance of the float32 comparisons."""
    from test_romepel_gpu import CONFIG_A, DECAY_RANK, romepel_tensors

    tensors = {k: v.double() for k, v in romepel_tensors(CONFIG_A, DECAY_RANK["A"], 66).items()}
    ids = helpers.token_ids(CONFIG_A["vocab"], 90, 4)
    good = plain.forward(CONFIG_A, tensors, ids)
    cfg = copy.deepcopy(CONFIG_A)
    keep = {n: getattr(plain, n) for n in ("distance_slopes", "query_temperature", "gla_walk", "positioned_embedding", "biased_attention")}
    if fault == "window":
        for layer in cfg["layers"]:
            if layer["type"] == "attention":
                layer["mixer"]["mask"]["size"] += 1
    elif fault == "slope":
        monkeypatch.setattr(plain, "distance_slopes", lambda h: keep["distance_slopes"](h) * 2.0 ** (-8.0 / h))
    elif fault == "temperature":
        monkeypatch.setattr(plain, "query_temperature", lambda p, c, e: keep["query_temperature"]([max(i - 1, 0) for i in p], c, e))
    elif fault == "position":
        monkeypatch.setattr(plain, "positioned_embedding", lambda i, t, p: keep["positioned_embedding"](i, t, torch.roll(p, 1, 0)))
    elif fault == "state":  # the state is lost once, in the middle
        monkeypatch.setattr(plain, "gla_walk", lambda q, k, v, a: torch.cat([keep["gla_walk"](q[:45], k[:45], v[:45], a[:45]),
                                                                             keep["gla_walk"](q[45:], k[45:], v[45:], a[45:])]))
    elif fault == "bias":
        tensors = dict(tensors)
        for name in [n for n in tensors if n.endswith("down.b")]:
            tensors[name] = torch.zeros_like(tensors[name])
    elif fault == "activation":
        tensors = dict(tensors)
        for name in [n for n in tensors if n.endswith(".act")]:
            tensors[name] = tensors[name].flip(0)
    else:
        monkeypatch.setattr(plain, "biased_attention", lambda q, k, v, *a: keep["biased_attention"](q, k.flip(1), v.flip(1), *a))
    bad = plain.forward(cfg, tensors, ids)
    off = ((bad - good) ** 2).mean(-1).sqrt() / (good ** 2).mean().sqrt()
    assert off.max() > 0.05, f"{fault}: {off.max():.3f}"
