"""Romepel: a decoder with learned position vectors whose layers mix tokens by windowed attention with a bias by
distance or by gated linear attention, each sublayer between two norms; which parts, in which order, from which
checkpoint tensors."""

from __future__ import annotations

from typing import List

from ..config.gilozen import GLA
from ..config.romepel import ATTENTION, RomepelConfig
from ..parts.base import make_part
from ..parts.embedding import LMHead, PositionedEmbedding
from ..weights.loader import ParamBinding, TensorSpec
from .gilozen import gla_mixer
from .registry import register_architecture
from .spec import LayerCall, ModelSpec, bind


def distance_slopes(heads: int) -> List[float]:
    """What head h takes off its scores for every position between query and key: 2^(-8 (h + 1) / heads)."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def build_romepel(cfg: RomepelConfig) -> ModelSpec:
    """x = embed[token] + pos[position]; layer i: x += norm1b(mixer(norm1(x))), then, if it has a feed-forward,
    x += norm2b(ff(norm2(x))); every norm is an RMS norm whose checkpoint tensor holds the factor less one.  Attention
    has biases on q, k and v and no rotation; the feed-forward is xIELU between two products with biases.  After the
    last layer the model's norm, the head, and the logits' soft cap.  Tensor names: ``embed``, ``pos``,
    ``l<i>.norm1`` ..., ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``; a bias is its weight's name + ``.b``."""
    w, eps = cfg.width, cfg.norm_eps
    bindings: List[ParamBinding] = []

    def norm(name: str):
        part = make_part("norm", "rms_norm", hidden_size=w, eps=eps, unit_offset=True)
        bind(bindings, part, "weight", [TensorSpec(name, (w,), "bias")])
        return part

    embedding = PositionedEmbedding(cfg.vocab, w, cfg.positions)
    bind(bindings, embedding, "weight", [TensorSpec("embed", (cfg.vocab, w))])
    bind(bindings, embedding, "position_weight", [TensorSpec("pos", (cfg.positions, w))])

    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.mix.", layer.mixer
        if layer.kind == ATTENTION:
            mixer = make_part("mixer", "gqa_attention", hidden_size=w, n_heads=m.heads, n_kv_heads=m.kv_heads,
                              head_dim=m.dim, value_dim=m.vdim, qkv_bias=True, position=make_part("position", "none"),
                              window=m.window, scale=m.scale, slopes=distance_slopes(m.heads),
                              query_temperature=m.temperature)
            rows = (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim))
            bind(bindings, mixer, "qkv_weight", [TensorSpec(p + name, (n, w)) for name, n in rows])
            bind(bindings, mixer, "qkv_bias", [TensorSpec(p + name + ".b", (n,), "bias") for name, n in rows])
            bind(bindings, mixer, "o_weight", [TensorSpec(p + "o", (w, m.heads * m.vdim))])
        elif layer.kind == GLA:
            mixer = gla_mixer(bindings, i, m, w, eps)
        else:  # pragma: no cover - the configuration has refused it
            raise ValueError(layer.kind)
        parts = dict(mixer_norm=norm(f"l{i}.norm1"), mixer=mixer, mixer_post_norm=norm(f"l{i}.norm1b"))
        if layer.ff is not None:
            ffn = make_part("feed_forward", "plain", hidden_size=w, intermediate_size=layer.ff, activation="xielu",
                            defer_bias=True)
            q = f"l{i}.mlp."
            bind(bindings, ffn, "up_weight", [TensorSpec(q + "up", (layer.ff, w))])
            bind(bindings, ffn, "up_bias", [TensorSpec(q + "up.b", (layer.ff,), "bias")])
            bind(bindings, ffn, "act", [TensorSpec(q + "act", (2,), "bias")])
            bind(bindings, ffn, "down_weight", [TensorSpec(q + "down", (w, layer.ff))])
            bind(bindings, ffn, "down_bias", [TensorSpec(q + "down.b", (w,), "bias")])
            parts.update(ffn_norm=norm(f"l{i}.norm2"), ffn=ffn, ffn_post_norm=norm(f"l{i}.norm2b"))
        layers.append(make_part("block", "sandwich_norm", **parts))
        schedule.append(LayerCall(i))

    final_norm = norm("final.norm")
    lm_head = LMHead(w, cfg.vocab, softcap=cfg.logit_softcap)
    bind(bindings, lm_head, "weight", [TensorSpec("head", (cfg.vocab, w))])
    # a layer without feed-forward may still carry the norms of one: not read
    unused = tuple(f"l{i}.{name}" for i, layer in enumerate(cfg.layers) if layer.ff is None for name in ("norm2", "norm2b"))
    return ModelSpec(config=cfg, embedding=embedding, layers=layers, schedule=schedule, final_norm=final_norm,
                     lm_head=lm_head, bindings=bindings, ignore_unexpected=unused)


register_architecture("Romepel", RomepelConfig, build_romepel)
