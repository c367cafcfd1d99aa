"""Typed configuration of the Mapedra decoder, read from its config.json.

The file names the model as ``"architecture": "Mapedra"`` and gives ``vocab``, ``width``, ``norm`` (``eps`` and ``groups``,
the equal parts a norm cuts its vector into; absent: 1), ``embedding.scale`` (the factor on the embedding's rows; absent:
1), ``token_side.dim`` (how many numbers of the side table every layer takes for a token) and a list ``layers``. Every
entry has a ``type`` (``lightning`` or ``attention``), the mixer's sizes and constants under ``mixer`` and its feed-forward
under ``mlp`` (``dense``, or null for none). Every size and constant is a key of the file; nothing has to be read from a
tensor's shape.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Dict, Mapping, Optional, Tuple, Union

from . import fields
from .fields import ConfigError, mapping, positive

LIGHTNING = "lightning"
ATTENTION = "attention"
DENSE = "dense"


@dataclass(frozen=True)
class BandScalingConfig:
    """Rotation rates stretched by how often they turn over ``original`` positions: by ``factor`` below ``low`` turns, not
    at all above ``high``, blended between."""
    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "BandScalingConfig":
        config = cls(**{name: fields.number(source, name) for name in ("factor", "low", "high", "original")})
        for name in ("factor", "low", "high", "original"):
            positive(getattr(config, name), f"mixer.rot.scaling.{name}")
        if config.high < config.low:
            raise ConfigError("mixer.rot.scaling.high must not lie below mixer.rot.scaling.low")
        return config

    def to_dict(self) -> Dict[str, Any]:
        return {"factor": self.factor, "high": self.high, "low": self.low, "original": self.original}


@dataclass(frozen=True)
class AttentionConfig:
    """Causal softmax attention with grouped key/value heads, norms of queries, keys and values, a rotation of
    neighbouring channels, a cap on the scores and a gate a channel."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    softcap: Optional[float] = None
    rot_scaling: Optional[BandScalingConfig] = None

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "AttentionConfig":
        rot = mapping(source, "rot")
        scaling = mapping(rot, "scaling", optional=True)
        config = cls(heads=fields.integer(source, "heads"), kv_heads=fields.integer(source, "kv_heads"),
                     dim=fields.integer(source, "dim"), vdim=fields.integer(source, "vdim"), scale=fields.number(source, "scale"),
                     rot_base=fields.number(rot, "base"), rot_dims=fields.integer(rot, "dims"),
                     softcap=fields.number(source, "softcap", None),
                     rot_scaling=BandScalingConfig.from_dict(scaling) if scaling is not None else None)
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("heads", "kv_heads", "dim", "vdim", "scale", "rot_base", "rot_dims"):
            positive(getattr(self, name), f"mixer.{name}")
        if self.heads % self.kv_heads != 0:
            raise ConfigError("mixer.heads must divide into mixer.kv_heads groups")
        if self.rot_dims % 2 != 0 or self.rot_dims > self.dim:
            raise ConfigError("mixer.rot.dims must be even and at most mixer.dim")
        if self.softcap is not None:
            positive(self.softcap, "mixer.softcap")

    def to_dict(self) -> Dict[str, Any]:
        rot: Dict[str, Any] = {"base": self.rot_base, "dims": self.rot_dims}
        if self.rot_scaling is not None:
            rot["scaling"] = self.rot_scaling.to_dict()
        out = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "rot": rot, "scale": self.scale, "vdim": self.vdim}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        return out


@dataclass(frozen=True)
class LightningConfig:
    """Linear attention with one fixed decay a head."""
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "LightningConfig":
        decay = source.get("decay")
        if not isinstance(decay, list) or not all(isinstance(value, (int, float)) and not isinstance(value, bool) for value in decay):
            raise ConfigError("config key decay must be a list of numbers")
        config = cls(heads=fields.integer(source, "heads"), dim=fields.integer(source, "dim"), vdim=fields.integer(source, "vdim"),
                     decay=tuple(float(value) for value in decay))
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("heads", "dim", "vdim"):
            positive(getattr(self, name), f"mixer.{name}")
        if len(self.decay) != self.heads:
            raise ConfigError("mixer.decay has one number a head")
        if not all(0.0 <= value <= 1.0 for value in self.decay):
            raise ConfigError("mixer.decay's numbers lie between 0 and 1")

    def to_dict(self) -> Dict[str, Any]:
        return {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class DenseMlpConfig:
    ff: int

    def to_dict(self) -> Dict[str, Any]:
        return {"ff": self.ff, "kind": DENSE}


def _mlp_from_dict(source: Optional[Mapping[str, Any]]) -> Optional[DenseMlpConfig]:
    if source is None:
        return None
    kind = fields.string(source, "kind")
    if kind != DENSE:
        raise ConfigError(f"unknown feed-forward kind {kind!r}; this design has {DENSE!r}")
    return DenseMlpConfig(ff=positive(fields.integer(source, "ff"), "mlp.ff"))


MixerConfig = Union[AttentionConfig, LightningConfig]
_MIXERS = {ATTENTION: AttentionConfig, LIGHTNING: LightningConfig}


@dataclass(frozen=True)
class MapedraLayerConfig:
    type: str
    mixer: MixerConfig
    mlp: Optional[DenseMlpConfig]

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "MapedraLayerConfig":
        kind = fields.string(source, "type")
        if kind not in _MIXERS:
            raise ConfigError(f"unknown layer type {kind!r}; this design has {', '.join(sorted(_MIXERS))}")
        return cls(type=kind, mixer=_MIXERS[kind].from_dict(mapping(source, "mixer")),
                   mlp=_mlp_from_dict(mapping(source, "mlp", optional=True)))

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None, "type": self.type}


@dataclass(frozen=True)
class MapedraConfig:
    vocab: int
    width: int
    norm_eps: float
    side_dim: int
    layers: Tuple[MapedraLayerConfig, ...]
    norm_groups: int = 1
    embedding_scale: float = 1.0
    architecture: str = "Mapedra"

    # what the engine's generic code asks of any configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "MapedraConfig":
        layers = source.get("layers")
        if not isinstance(layers, list) or not layers or not all(isinstance(layer, dict) for layer in layers):
            raise ConfigError("config key layers must be a list of objects with at least one entry")
        norm = mapping(source, "norm")
        config = cls(vocab=fields.integer(source, "vocab"), width=fields.integer(source, "width"),
                     norm_eps=fields.number(norm, "eps"), norm_groups=fields.integer(norm, "groups", 1),
                     side_dim=fields.integer(mapping(source, "token_side"), "dim"),
                     embedding_scale=fields.number(mapping(source, "embedding", optional=True) or {}, "scale", 1.0),
                     layers=tuple(MapedraLayerConfig.from_dict(layer) for layer in layers),
                     architecture=fields.string(source, "architecture", "Mapedra"))
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("vocab", "width", "norm_eps", "norm_groups", "side_dim"):
            positive(getattr(self, name), name)
        if self.width % self.norm_groups != 0:
            raise ConfigError("width must divide into norm.groups equal parts")

    def to_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                "layers": [layer.to_dict() for layer in self.layers], "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
                "token_side": {"dim": self.side_dim}, "vocab": self.vocab, "width": self.width}

    def save(self, folder: str) -> None:
        os.makedirs(folder, exist_ok=True)
        with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as handle:
            json.dump(self.to_dict(), handle, indent=1, sort_keys=True)
