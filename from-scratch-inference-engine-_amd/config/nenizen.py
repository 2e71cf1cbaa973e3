"""Configuration of the Nenizen decoder (config.json ``"architecture": "Nenizen"``): a list of layers, each with attention
through a latent of one of three kinds and an optional feed-forward (dense with a clipped gate, or routed experts beside
a shared one), a norm before and after every sublayer, a run of layers that is passed several times, and soft-capped
logits."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from .base import ConfigError, ModelConfig, checked_float, checked_int, end_token_of, required_int


@dataclass(frozen=True)
class LatentKind:
    """What tells the mixers apart: whether queries go through a latent of their own, which values the rotation pairs,
    whether a window bounds what a query sees, whether the softmax has a sink a head, and what the gate multiplies
    (every value, every head, nothing)."""

    query_latent: bool
    layout: str
    window: bool
    sink: bool
    gate: Optional[str]


KINDS = {
    "latent_attention": LatentKind(query_latent=False, layout="interleaved", window=False, sink=False, gate="values"),
    "latent_attention_2": LatentKind(query_latent=True, layout="half", window=True, sink=False, gate="heads"),
    "latent_attention_3": LatentKind(query_latent=True, layout="half", window=False, sink=True, gate=None),
}
DENSE, EXPERTS = "dense", "moe"


def _object(raw: Mapping, key: str, where: str) -> Mapping:
    if not isinstance(raw.get(key), dict):
        raise ConfigError(f"config.json: {where} has no object '{key}'")
    return raw[key]


def _size(raw: Mapping, key: str, where: str, minimum: int = 1) -> int:
    if key not in raw:
        raise ConfigError(f"config.json: {where} has no '{key}'")
    return checked_int(raw[key], f"{where}.{key}", minimum)


@dataclass(frozen=True)
class LatentAttentionConfig:
    """``dim`` unrotated and ``rot_dim`` rotated query/key values a head, values of ``vdim``, a key/value latent of
    ``kv_rank``, a query latent of ``q_rank`` (None: the kind has none), ``window`` positions (None: all before)."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    q_rank: Optional[int] = None
    window: Optional[int] = None

    @classmethod
    def from_mixer(cls, m: Mapping, kind: LatentKind, where: str) -> "LatentAttentionConfig":
        rot_dim = _size(m, "rot_dim", where, 0)
        rot = _object(m, "rot", where)
        if rot_dim % 2 or _size(rot, "dims", where + ".rot", 0) != rot_dim:
            raise ConfigError(f"config.json: {where}: rot.dims must be rot_dim {rot_dim}, and that even")
        return cls(heads=_size(m, "heads", where), dim=_size(m, "dim", where), rot_dim=rot_dim, vdim=_size(m, "vdim", where),
                   kv_rank=_size(m, "kv_rank", where), scale=checked_float(m.get("scale"), f"{where}.scale"),
                   rot_base=checked_float(rot.get("base"), f"{where}.rot.base"),
                   q_rank=_size(m, "q_rank", where) if kind.query_latent else None,
                   window=_size(_object(m, "mask", where), "size", where + ".mask") if kind.window else None)

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "kv_rank": self.kv_rank,
             "scale": self.scale, "rot": {"base": self.rot_base, "dims": self.rot_dim}}
        if self.q_rank is not None:
            d["q_rank"] = self.q_rank
        if self.window is not None:
            d["mask"] = {"size": self.window}
        return d


@dataclass(frozen=True)
class FeedForwardConfig:
    """``kind`` DENSE: one of width ``ff`` whose gate and up values are cut off at ``limit``.  EXPERTS: ``experts`` of width
    ``ff`` of which a token uses ``top``, and one of width ``shared_ff`` for every token (None: none)."""

    kind: str
    ff: int
    limit: float = 0.0
    experts: int = 0
    top: int = 0
    shared_ff: Optional[int] = None

    @classmethod
    def from_mlp(cls, mlp: Mapping, where: str) -> "FeedForwardConfig":
        kind = mlp.get("kind")
        if kind == DENSE:
            return cls(DENSE, _size(mlp, "ff", where), limit=checked_float(mlp.get("limit"), f"{where}.limit"))
        if kind != EXPERTS:
            raise ConfigError(f"config.json: {where}.kind '{kind}' is not a feed-forward of this architecture ({DENSE}, {EXPERTS})")
        router = _object(mlp, "router", where)
        experts = _size(router, "experts", where + ".router")
        top = _size(router, "top", where + ".router")
        if top > experts:
            raise ConfigError(f"config.json: {where}.router: top {top} of {experts} experts")
        shared = None if mlp.get("shared") is None else _size(_object(mlp, "shared", where), "ff", where + ".shared")
        return cls(EXPERTS, _size(_object(mlp, "expert", where), "ff", where + ".expert"), experts=experts, top=top,
                   shared_ff=shared)

    def to_dict(self) -> dict:
        if self.kind == DENSE:
            return {"kind": DENSE, "ff": self.ff, "limit": self.limit}
        d = {"kind": EXPERTS, "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclass(frozen=True)
class LayerConfig:
    kind: str  # a key of KINDS
    mixer: LatentAttentionConfig
    mlp: Optional[FeedForwardConfig]  # None: the layer has none

    def to_dict(self) -> dict:
        return {"type": self.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class LoopConfig:
    """Layers ``start`` .. ``stop`` - 1 run ``times`` times in a row."""

    start: int
    stop: int
    times: int

    def to_dict(self) -> dict:
        return {"start": self.start, "stop": self.stop, "times": self.times}


@dataclass(frozen=True)
class NenizenConfig(ModelConfig):
    width: int = 0
    vocab: int = 0
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    logit_softcap: Optional[float] = None
    layers: Tuple[LayerConfig, ...] = ()
    loop: Optional[LoopConfig] = None
    eos_token_id: int = -1

    @property
    def end_token(self) -> int:
        return self.eos_token_id

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "NenizenConfig":
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(layers_raw):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"config.json: {where} must be an object with a 'mixer'")
            kind = entry.get("type")
            if kind not in KINDS:
                raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this architecture ({', '.join(KINDS)})")
            mlp = entry.get("mlp")
            if mlp is not None and not isinstance(mlp, dict):
                raise ConfigError(f"config.json: {where}.mlp must be null or an object")
            layers.append(LayerConfig(kind, LatentAttentionConfig.from_mixer(entry["mixer"], KINDS[kind], where),
                                      None if mlp is None else FeedForwardConfig.from_mlp(mlp, where + ".mlp")))
        loop = None
        if raw.get("loop") is not None:
            entry = _object(raw, "loop", "the model")
            loop = LoopConfig(_size(entry, "start", "loop", 0), _size(entry, "stop", "loop"), _size(entry, "times", "loop"))
            if not loop.start < loop.stop <= len(layers):
                raise ConfigError(f"config.json: loop from {loop.start} to {loop.stop} does not lie within {len(layers)} layers")
        norm, embedding, cap = raw.get("norm") or {}, raw.get("embedding") or {}, raw.get("logit_softcap")
        return cls(architecture="Nenizen", width=required_int(raw, "width"), vocab=required_int(raw, "vocab"),
                   norm_eps=checked_float(norm.get("eps", 1e-6), "norm.eps", positive=False),
                   embedding_scale=checked_float(embedding.get("scale", 1.0), "embedding.scale"),
                   logit_softcap=None if cap is None else checked_float(cap, "logit_softcap"),
                   layers=tuple(layers), loop=loop, eos_token_id=end_token_of(raw))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "width": self.width, "vocab": self.vocab, "norm": {"eps": self.norm_eps},
             "embedding": {"scale": self.embedding_scale}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        if self.eos_token_id >= 0:
            d["eos_token_id"] = self.eos_token_id
        return d
