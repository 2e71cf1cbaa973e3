"""Nenizen: a decoder of attention through latents whose middle layers are passed several times with the same weights;
which parts, in which order, from which checkpoint tensors."""

from __future__ import annotations

from typing import List

from .. import ops
from ..config.nenizen import DENSE, KINDS, FeedForwardConfig, NenizenConfig
from ..parts.base import make_part
from ..parts.embedding import LMHead, TokenEmbedding
from ..weights.loader import ParamBinding, TensorSpec
from .registry import register_architecture
from .spec import LayerCall, ModelSpec, bind

GATE_SLOPE = 1.702  # of the sigmoid of the dense feed-forward's clipped gate


def build_nenizen(cfg: NenizenConfig) -> ModelSpec:
    """x = embed[token] * scale; layer i: x += norm1b(mixer(norm1(x))), then, if it has a feed-forward,
    x += norm2b(ff(norm2(x))), all RMS norms with a plain weight.  Before each pass of the loop's layers the stream becomes
    ``loop.in`` [x; x0] + ``loop.step``[pass], x0 the embedding's output; every pass has caches of its own.  After the last
    layer the model's norm, the head, which is the embedding table, and the logits' soft cap.  Tensor names: ``embed``,
    ``loop.*``, ``l<i>.norm1`` ..., ``l<i>.mix.*``, ``l<i>.mlp.*`` (an expert's matrices are ``l<i>.mlp.e<j>.gate``, ``.up``
    and ``.down``, the shared one's ``l<i>.mlp.shared.*``), ``final.norm``."""
    w, eps = cfg.width, cfg.norm_eps
    bindings: List[ParamBinding] = []

    def norm(name: str):
        part = make_part("norm", "rms_norm", hidden_size=w, eps=eps)
        bind(bindings, part, "weight", [TensorSpec(name, (w,), "norm")])
        return part

    def gated(p: str, ff: int, activation):
        part = make_part("feed_forward", "gated", hidden_size=w, intermediate_size=ff, activation=activation)
        bind(bindings, part, "gate_up_weight", [TensorSpec(p + "gate", (ff, w)), TensorSpec(p + "up", (ff, w))])
        bind(bindings, part, "down_weight", [TensorSpec(p + "down", (w, ff))])
        return part

    def feed_forward(p: str, e: FeedForwardConfig):
        if e.kind == DENSE:
            return gated(p, e.ff, ops.GateAct("clipped", limit=e.limit, slope=GATE_SLOPE))
        part = make_part("feed_forward", "routed_experts", hidden_size=w, intermediate_size=e.ff, n_experts=e.experts, top=e.top,
                         scores="softmax", renorm=False, correction=False, gated="silu",
                         shared=None if e.shared_ff is None else gated(p + "shared.", e.shared_ff, "silu"))
        bind(bindings, part, "router_weight", [TensorSpec(p + "router", (e.experts, w))])
        bind(bindings, part, "up_weight", [TensorSpec(f"{p}e{j}.{name}", (e.ff, w)) for j in range(e.experts)
                                           for name in ("gate", "up")])
        bind(bindings, part, "down_weight", [TensorSpec(f"{p}e{j}.down", (w, e.ff)) for j in range(e.experts)])
        return part

    embedding = TokenEmbedding(cfg.vocab, w, scale=cfg.embedding_scale)
    embed_spec = TensorSpec("embed", (cfg.vocab, w))
    bind(bindings, embedding, "weight", [embed_spec])

    layers = []
    for i, layer in enumerate(cfg.layers):
        p, m, kind = f"l{i}.mix.", layer.mixer, KINDS[layer.kind]
        position = make_part("position", "rope", head_dim=m.rot_dim, theta=m.rot_base, layout=kind.layout) if m.rot_dim \
            else make_part("position", "none")
        mixer = make_part("mixer", "latent_attention", hidden_size=w, n_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim,
                          value_dim=m.vdim, kv_rank=m.kv_rank, q_rank=m.q_rank, scale=m.scale, norm_eps=eps, position=position,
                          sink=kind.sink, gate=kind.gate, window=m.window)
        q_size = m.heads * (m.dim + m.rot_dim)
        down = [TensorSpec(p + "q", (q_size, w)) if m.q_rank is None else TensorSpec(p + "dq", (m.q_rank, w)),
                TensorSpec(p + "dkv", (m.kv_rank + m.rot_dim, w))]
        if kind.gate is not None:
            down.append(TensorSpec(p + "g", (m.heads if kind.gate == "heads" else m.heads * m.vdim, w)))
        bind(bindings, mixer, "down_weight", down)
        if m.q_rank is not None:
            bind(bindings, mixer, "q_norm_weight", [TensorSpec(p + "dq.norm", (m.q_rank,), "norm")])
            bind(bindings, mixer, "uq_weight", [TensorSpec(p + "uq", (q_size, m.q_rank))])
        bind(bindings, mixer, "kv_norm_weight", [TensorSpec(p + "dkv.norm", (m.kv_rank,), "norm")])
        bind(bindings, mixer, "uk_weight", [TensorSpec(p + "uk", (m.heads * m.dim, m.kv_rank))])
        bind(bindings, mixer, "uv_weight", [TensorSpec(p + "uv", (m.heads * m.vdim, m.kv_rank))])
        if kind.sink:
            bind(bindings, mixer, "sink", [TensorSpec(p + "sink", (m.heads,), "bias")])
        bind(bindings, mixer, "o_weight", [TensorSpec(p + "o", (w, m.heads * m.vdim))])
        parts = dict(mixer_norm=norm(f"l{i}.norm1"), mixer=mixer, mixer_post_norm=norm(f"l{i}.norm1b"))
        if layer.mlp is not None:
            parts.update(ffn_norm=norm(f"l{i}.norm2"), ffn=feed_forward(f"l{i}.mlp.", layer.mlp),
                         ffn_post_norm=norm(f"l{i}.norm2b"))
        layers.append(make_part("block", "sandwich_norm", **parts))

    schedule, loop = [], cfg.loop
    if loop is None:
        schedule = [LayerCall(i) for i in range(len(layers))]
    else:
        entrance = make_part("entrance", "origin_mix", hidden_size=w, numbers=loop.times)
        bind(bindings, entrance, "weight", [TensorSpec("loop.in", (w, 2 * w))])
        bind(bindings, entrance, "step", [TensorSpec("loop.step", (loop.times, w), "bias")])
        schedule = [LayerCall(i) for i in range(loop.start)]
        for t in range(loop.times):
            schedule.append(LayerCall(loop.start, entrance=entrance, entrance_number=t))
            schedule += [LayerCall(i) for i in range(loop.start + 1, loop.stop)]
        schedule += [LayerCall(i) for i in range(loop.stop, len(layers))]

    final_norm = norm("final.norm")
    lm_head = LMHead(w, cfg.vocab, softcap=cfg.logit_softcap)
    bind(bindings, lm_head, "weight", [embed_spec])
    # a layer without feed-forward may still carry the norms of one: not read
    unused = tuple(f"l{i}.{name}" for i, layer in enumerate(cfg.layers) if layer.mlp is None for name in ("norm2", "norm2b"))
    return ModelSpec(config=cfg, embedding=embedding, layers=layers, schedule=schedule, final_norm=final_norm,
                     lm_head=lm_head, bindings=bindings, ignore_unexpected=unused)


register_architecture("Nenizen", NenizenConfig, build_nenizen)
