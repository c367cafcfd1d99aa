"""Typed configuration of the Zuluvik decoder, read from its config.json.

The file names the model as ``"architecture": "Zuluvik"`` and gives ``vocab``, ``width``, ``norm.eps``,
``embedding.scale`` (the factor on the embedding's rows; absent: 1) and a list ``layers``. Every entry has a ``type``
(``attention``, ``attention_2`` or ``latent_attention``), the mixer's sizes and constants under ``mixer`` and its
feed-forward under ``mlp`` (``moe``, or null for none). An entry with ``weights_of`` names another layer, whose tensors it
runs with; the rest of the entry says the same as that layer's. Every size and constant is a key of the file; nothing has
to be read from a tensor's shape.
"""
from __future__ import annotations

import json
import math
import os
from dataclasses import dataclass
from typing import Any, Dict, Mapping, Optional, Tuple, Union

from . import fields
from .fields import ConfigError, mapping, positive

DIFFERENTIAL_ATTENTION = "attention"
ROTARY_ATTENTION = "attention_2"
LATENT_ATTENTION = "latent_attention"
MOE = "moe"


@dataclass(frozen=True)
class RampScalingConfig:
    """Rotation rates stretched by ``factor`` where a pair turns seldom over ``original`` positions (``slow`` times or
    fewer), left where it turns often (``fast`` times or more), blended along the pairs between."""
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "RampScalingConfig":
        config = cls(**{name: fields.number(source, name) for name in ("factor", "original", "fast", "slow")})
        for name in ("factor", "original", "fast", "slow"):
            positive(getattr(config, name), f"mixer.rot.scaling.{name}")
        return config

    def to_dict(self) -> Dict[str, Any]:
        return {"factor": self.factor, "fast": self.fast, "original": self.original, "slow": self.slow}


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int
    scaling: Optional[RampScalingConfig] = None

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "RotationConfig":
        scaling = mapping(source, "scaling", optional=True)
        config = cls(base=fields.number(source, "base"), dims=fields.integer(source, "dims"),
                     scaling=RampScalingConfig.from_dict(scaling) if scaling is not None else None)
        positive(config.base, "mixer.rot.base")
        positive(config.dims, "mixer.rot.dims")
        if config.dims % 2 != 0:
            raise ConfigError("mixer.rot.dims must be even")
        if config.scaling is not None and math.log(config.base) == 0.0:
            raise ConfigError("mixer.rot.base must not be 1 where rates are stretched")
        return config

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = self.scaling.to_dict()
        return out


@dataclass(frozen=True)
class DifferentialAttentionConfig:
    """Causal attention of two maps a head over the same values, whose difference counts; a short convolution over time
    on queries, keys and values; no rotation."""
    heads: int
    kv_heads: int
    dim: int            # query/key dims of one map of a head
    vdim: int
    conv: int
    diff: float
    scale: float

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "DifferentialAttentionConfig":
        config = cls(**{name: fields.integer(source, name) for name in ("heads", "kv_heads", "dim", "vdim", "conv")},
                     diff=fields.number(source, "diff"), scale=fields.number(source, "scale"))
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("heads", "kv_heads", "dim", "vdim", "conv"):
            positive(getattr(self, name), f"mixer.{name}")
        if self.heads % self.kv_heads != 0:
            raise ConfigError("mixer.heads must divide into mixer.kv_heads groups")

    def to_dict(self) -> Dict[str, Any]:
        return {"conv": self.conv, "diff": self.diff, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class RotaryAttentionConfig:
    """Causal attention with biases on queries, keys and values, a rotation of neighbouring channels, and a norm of the
    turned queries and keys without a weight."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotationConfig

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "RotaryAttentionConfig":
        config = cls(**{name: fields.integer(source, name) for name in ("heads", "kv_heads", "dim", "vdim")},
                     scale=fields.number(source, "scale"), rot=RotationConfig.from_dict(mapping(source, "rot")))
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("heads", "kv_heads", "dim", "vdim"):
            positive(getattr(self, name), f"mixer.{name}")
        if self.heads % self.kv_heads != 0:
            raise ConfigError("mixer.heads must divide into mixer.kv_heads groups")
        if self.rot.dims > self.dim:
            raise ConfigError("mixer.rot.dims must be at most mixer.dim")

    def to_dict(self) -> Dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "rot": self.rot.to_dict(), "scale": self.scale,
                "vdim": self.vdim}


@dataclass(frozen=True)
class LatentAttentionConfig:
    """Causal attention whose keys and values are projected up from one cached latent vector a token; the queries come
    straight from the input; the rotated parts turn with neighbouring channels paired."""
    heads: int
    dim: int            # unrotated query/key dims a head
    rot_dim: int        # rotated query/key dims a head; the keys' rotated part is shared by all heads
    vdim: int
    kv_rank: int
    scale: float
    rot: RotationConfig

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "LatentAttentionConfig":
        config = cls(**{name: fields.integer(source, name) for name in ("heads", "dim", "rot_dim", "vdim", "kv_rank")},
                     scale=fields.number(source, "scale"), rot=RotationConfig.from_dict(mapping(source, "rot")))
        config.validate()
        return config

    def validate(self) -> None:
        for name in ("heads", "dim", "rot_dim", "vdim", "kv_rank"):
            positive(getattr(self, name), f"mixer.{name}")
        if self.rot.dims != self.rot_dim:
            raise ConfigError("mixer.rot.dims must equal mixer.rot_dim: the rotated part turns whole")

    def to_dict(self) -> Dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "rot": self.rot.to_dict(), "rot_dim": self.rot_dim,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class ExpertConfig:
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, source: Mapping[str, Any], where: str) -> "ExpertConfig":
        return cls(ff=positive(fields.integer(source, "ff"), f"{where}.ff"), limit=positive(fields.number(source, "limit"), f"{where}.limit"))

    def to_dict(self) -> Dict[str, Any]:
        return {"ff": self.ff, "limit": self.limit}


@dataclass(frozen=True)
class MoeMlpConfig:
    experts: int
    top: int
    expert: ExpertConfig
    identity: int = 0           # router outputs after the experts' that return their input
    groups: int = 1             # router.groups.count, over experts and identity places; 1: every one can be chosen
    keep_groups: int = 1        # router.groups.keep
    scale: float = 1.0          # router.scale
    shared: Optional[ExpertConfig] = None

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "MoeMlpConfig":
        router = mapping(source, "router")
        groups = mapping(router, "groups", optional=True)
        shared = mapping(source, "shared", optional=True)
        config = cls(experts=fields.integer(router, "experts"), top=fields.integer(router, "top"),
                     expert=ExpertConfig.from_dict(mapping(source, "expert"), "mlp.expert"),
                     identity=fields.integer(router, "identity", 0),
                     groups=fields.integer(groups, "count") if groups is not None else 1,
                     keep_groups=fields.integer(groups, "keep") if groups is not None else 1,
                     scale=fields.number(router, "scale", 1.0),
                     shared=ExpertConfig.from_dict(shared, "mlp.shared") if shared is not None else None)
        config.validate()
        return config

    @property
    def places(self) -> int:
        return self.experts + self.identity

    def validate(self) -> None:
        for name in ("experts", "top", "groups", "keep_groups"):
            positive(getattr(self, name), f"mlp.router.{name}")
        if self.identity < 0:
            raise ConfigError("mlp.router.identity must not be negative")
        if self.top > self.places:
            raise ConfigError("mlp.router.top cannot exceed the experts and identity places")
        if self.places % self.groups != 0 or self.keep_groups > self.groups:
            raise ConfigError("mlp.router.groups: equal groups of experts and identity places, of which at most all are kept")
        if self.keep_groups * (self.places // self.groups) < self.top:
            raise ConfigError("mlp.router.groups: the kept groups hold fewer places than a token takes")

    def to_dict(self) -> Dict[str, Any]:
        router: Dict[str, Any] = {"experts": self.experts, "groups": {"count": self.groups, "keep": self.keep_groups},
                                  "identity": self.identity, "scale": self.scale, "top": self.top}
        out: Dict[str, Any] = {"expert": self.expert.to_dict(), "kind": MOE, "router": router}
        if self.shared is not None:
            out["shared"] = self.shared.to_dict()
        return out


def _mlp_from_dict(source: Optional[Mapping[str, Any]]) -> Optional[MoeMlpConfig]:
    if source is None:
        return None
    kind = fields.string(source, "kind")
    if kind != MOE:
        raise ConfigError(f"unknown feed-forward kind {kind!r}; this design has {MOE!r}")
    return MoeMlpConfig.from_dict(source)


MixerConfig = Union[DifferentialAttentionConfig, RotaryAttentionConfig, LatentAttentionConfig]
_MIXERS = {DIFFERENTIAL_ATTENTION: DifferentialAttentionConfig, ROTARY_ATTENTION: RotaryAttentionConfig,
           LATENT_ATTENTION: LatentAttentionConfig}


@dataclass(frozen=True)
class ZuluvikLayerConfig:
    type: str
    mixer: MixerConfig
    mlp: Optional[MoeMlpConfig]
    weights_of: Optional[int] = None    # the layer whose tensors this one runs with

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "ZuluvikLayerConfig":
        kind = fields.string(source, "type")
        if kind not in _MIXERS:
            raise ConfigError(f"unknown layer type {kind!r}; this design has {', '.join(sorted(_MIXERS))}")
        return cls(type=kind, mixer=_MIXERS[kind].from_dict(mapping(source, "mixer")),
                   mlp=_mlp_from_dict(mapping(source, "mlp", optional=True)), weights_of=fields.integer(source, "weights_of", None))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None, "type": self.type}
        if self.weights_of is not None:
            out["weights_of"] = self.weights_of
        return out


@dataclass(frozen=True)
class ZuluvikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[ZuluvikLayerConfig, ...]
    embedding_scale: float = 1.0
    architecture: str = "Zuluvik"

    # what the engine's generic code asks of any configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "ZuluvikConfig":
        layers = source.get("layers")
        if not isinstance(layers, list) or not layers or not all(isinstance(layer, dict) for layer in layers):
            raise ConfigError("config key layers must be a list of objects with at least one entry")
        embedding = mapping(source, "embedding", optional=True)
        config = cls(vocab=fields.integer(source, "vocab"), width=fields.integer(source, "width"),
                     norm_eps=fields.number(mapping(source, "norm"), "eps"),
                     layers=tuple(ZuluvikLayerConfig.from_dict(layer) for layer in layers),
                     embedding_scale=fields.number(embedding, "scale", 1.0) if embedding is not None else 1.0,
                     architecture=fields.string(source, "architecture", "Zuluvik"))
        config.validate()
        return config

    def validate(self) -> None:
        positive(self.vocab, "vocab")
        positive(self.width, "width")
        positive(self.norm_eps, "norm.eps")
        for index, layer in enumerate(self.layers):
            if layer.weights_of is None:
                continue
            if not 0 <= layer.weights_of < len(self.layers):
                raise ConfigError(f"layers[{index}].weights_of names no layer")
            owner = self.layers[self.owner_of(index)]
            if (layer.type, layer.mixer, layer.mlp) != (owner.type, owner.mixer, owner.mlp):
                raise ConfigError(f"layers[{index}] differs from the layer whose weights it runs with")

    def owner_of(self, index: int) -> int:
        """The layer whose tensors layer ``index`` runs with: itself, or where ``weights_of`` leads."""
        seen = set()
        while self.layers[index].weights_of is not None:
            if index in seen or not 0 <= self.layers[index].weights_of < len(self.layers):
                raise ConfigError(f"layers[{index}].weights_of leads to no layer with tensors of its own")
            seen.add(index)
            index = self.layers[index].weights_of
        return index

    def to_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                "layers": [layer.to_dict() for layer in self.layers], "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}

    def save(self, folder: str) -> None:
        os.makedirs(folder, exist_ok=True)
        with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as handle:
            json.dump(self.to_dict(), handle, indent=1, sort_keys=True)
