"""Configuration of the Romepel decoder (config.json ``"architecture": "Romepel"``): learned position vectors, a list
of layers, each with a mixer of one of two kinds (grouped-query attention over a window with a bias by distance and
queries scaled by their position, gated linear attention) and an optional feed-forward without a gate, a norm before
and after every sublayer, and soft-capped logits."""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any, Mapping, Optional, Tuple

from .base import ConfigError, ModelConfig, checked_float, checked_int, end_token_of, required_int
from .gilozen import GLA, GLAConfig, with_decay_ranks

ATTENTION = "attention"


@dataclass(frozen=True)
class AttentionConfig:
    """``heads`` query and ``kv_heads`` key/value heads, queries and keys of ``dim`` and values of ``vdim``; a query
    sees itself and the ``window`` - 1 positions before it (None: all).  ``temperature`` = (coef, every): queries at
    position p are multiplied by 1 + coef ln(floor((p + 1) / every) + 1) (None: as they are)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None
    temperature: Optional[Tuple[float, float]] = None

    @classmethod
    def from_mixer(cls, m: Mapping, where: str) -> "AttentionConfig":
        def size(key):
            if key not in m:
                raise ConfigError(f"config.json: {where} has no '{key}'")
            return checked_int(m[key], f"{where}.{key}", 1)

        window = temperature = None
        if m.get("mask") is not None:
            if not isinstance(m["mask"], dict):
                raise ConfigError(f"config.json: {where}.mask must be an object with a 'size'")
            window = checked_int(m["mask"].get("size"), f"{where}.mask.size", 1)
        if m.get("q_temp") is not None:
            if not isinstance(m["q_temp"], dict):
                raise ConfigError(f"config.json: {where}.q_temp must be an object with 'coef' and 'every'")
            temperature = (checked_float(m["q_temp"].get("coef"), f"{where}.q_temp.coef", positive=False),
                           checked_float(m["q_temp"].get("every"), f"{where}.q_temp.every"))
        mixer = cls(heads=size("heads"), kv_heads=size("kv_heads"), dim=size("dim"), vdim=size("vdim"),
                    scale=checked_float(m.get("scale"), f"{where}.scale"), window=window, temperature=temperature)
        if mixer.heads % mixer.kv_heads:
            raise ConfigError(f"config.json: {where}: heads {mixer.heads} must be a multiple of kv_heads {mixer.kv_heads}")
        return mixer

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        if self.temperature is not None:
            d["q_temp"] = {"coef": self.temperature[0], "every": self.temperature[1]}
        return d


@dataclass(frozen=True)
class LayerConfig:
    kind: str          # ATTENTION or GLA
    mixer: object      # AttentionConfig or GLAConfig
    ff: Optional[int]  # width of the feed-forward, None: the layer has none

    def to_dict(self) -> dict:
        return {"type": self.kind, "mixer": self.mixer.to_dict(),
                "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


@dataclass(frozen=True)
class RomepelConfig(ModelConfig):
    width: int = 0
    vocab: int = 0
    positions: int = 0
    norm_eps: float = 1e-6
    logit_softcap: Optional[float] = None
    layers: Tuple[LayerConfig, ...] = ()
    eos_token_id: int = -1

    @property
    def max_positions(self) -> int:
        return self.positions

    @property
    def end_token(self) -> int:
        return self.eos_token_id

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "RomepelConfig":
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(layers_raw):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"config.json: {where} must be an object with a 'mixer'")
            kind = entry.get("type")
            if kind == ATTENTION:
                mixer = AttentionConfig.from_mixer(entry["mixer"], where)
            elif kind == GLA:
                mixer = GLAConfig.from_mixer(entry["mixer"], where)
            else:
                raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this architecture "
                                  f"({ATTENTION}, {GLA})")
            mlp, ff = entry.get("mlp"), None
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind", "dense") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp must be null or a dense feed-forward")
                ff = checked_int(mlp.get("ff"), f"{where}.mlp.ff", 1)
            layers.append(LayerConfig(kind, mixer, ff))
        norm = raw.get("norm") or {}
        cap = raw.get("logit_softcap")
        return cls(architecture="Romepel", width=required_int(raw, "width"), vocab=required_int(raw, "vocab"),
                   positions=required_int(raw, "max_positions"),
                   norm_eps=checked_float(norm.get("eps", 1e-6), "norm.eps", positive=False),
                   logit_softcap=None if cap is None else checked_float(cap, "logit_softcap"),
                   layers=tuple(layers), eos_token_id=end_token_of(raw))

    def completed_from(self, tensor_shapes: Mapping[str, tuple]) -> "RomepelConfig":
        return replace(self, layers=with_decay_ranks(self.layers, tensor_shapes))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "width": self.width, "vocab": self.vocab, "max_positions": self.positions,
             "norm": {"eps": self.norm_eps}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        if self.eos_token_id >= 0:
            d["eos_token_id"] = self.eos_token_id
        return d
