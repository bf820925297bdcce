"""Typed configuration of the Sorovik decoder.

config.json names the vocabulary, the width, one eps for every norm and a list of layers.  Every layer names its mixer
(`type`: "latent_attention" or "attention"), the mixer's sizes (`mixer`) and its feed-forward (`mlp`, null for none;
`kind` "dense" or "moe").  Strict as every configuration: an unknown key is an error that names it.
"""

from __future__ import annotations

import re
from dataclasses import dataclass
from typing import Any, List, Mapping, Optional

from .schema import ConfigError, from_dict


@dataclass(frozen=True)
class NormConfig:
    eps: float

    def __post_init__(self) -> None:
        if self.eps <= 0:
            raise ConfigError("norm.eps must be positive")


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int

    def __post_init__(self) -> None:
        if self.dims < 0 or self.dims % 2 != 0:
            raise ConfigError("rot.dims must be even and not negative")
        if self.base <= 0:
            raise ConfigError("rot.base must be positive")


@dataclass(frozen=True)
class WindowConfig:
    size: int  # keys a query reads, its own included

    def __post_init__(self) -> None:
        if self.size < 1:
            raise ConfigError("mask.size must be at least 1")


@dataclass(frozen=True)
class KeptWindowConfig(WindowConfig):
    keep_first: int = 0  # keys at the sequence's start that every query reads besides

    def __post_init__(self) -> None:
        super().__post_init__()
        if self.keep_first < 0:
            raise ConfigError("mask.keep_first cannot be negative")


@dataclass(frozen=True)
class LatentAttentionConfig:
    """`heads` heads with `dim` unrotated and `rot_dim` rotated query/key dimensions and values of `vdim`, keys and values
    from a latent of `kv_rank`.  `kv_from`: the layer whose cached rows this layer reads instead of making its own."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: Optional[RotationConfig] = None
    mask: Optional[WindowConfig] = None
    kv_from: Optional[int] = None

    def __post_init__(self) -> None:
        if min(self.heads, self.dim, self.vdim, self.kv_rank) < 1 or self.rot_dim < 0 or self.rot_dim % 2 != 0:
            raise ConfigError("a latent attention's sizes must be positive, and rot_dim even")
        if self.rot is not None and self.rot.dims > self.rot_dim:
            raise ConfigError(f"rot.dims {self.rot.dims} exceeds rot_dim {self.rot_dim}")
        if self.scale <= 0:
            raise ConfigError("scale must be positive")


@dataclass(frozen=True)
class AttentionConfig:
    """`heads` query heads on `kv_heads` key/value heads of `dim` elements (the values are the keys, so `vdim` is `dim`);
    `conv`: inputs that the convolution on queries and keys reads, the current one included (None: no convolution)."""

    heads: int
    kv_heads: int
    dim: int
    scale: float
    vdim: Optional[int] = None
    conv: Optional[int] = None
    rot: Optional[RotationConfig] = None
    mask: Optional[KeptWindowConfig] = None

    def __post_init__(self) -> None:
        if min(self.heads, self.kv_heads, self.dim) < 1:
            raise ConfigError("an attention mixer's sizes must be positive")
        if self.heads % self.kv_heads != 0:
            raise ConfigError(f"{self.heads} query heads do not divide into {self.kv_heads} key/value heads")
        if self.vdim is not None and self.vdim != self.dim:
            raise ConfigError(f"the values are the keys: vdim {self.vdim} must equal dim {self.dim}")
        if self.conv is not None and self.conv < 1:
            raise ConfigError("conv must be at least 1")
        if self.rot is not None and self.rot.dims > self.dim:
            raise ConfigError(f"rot.dims {self.rot.dims} exceeds the head's {self.dim} dimensions")
        if self.scale <= 0:
            raise ConfigError("scale must be positive")


@dataclass(frozen=True)
class GroupsConfig:
    count: int  # equal groups of neighbouring experts
    keep: int  # groups that stay open to a token's choice

    def __post_init__(self) -> None:
        if not 1 <= self.keep <= self.count:
            raise ConfigError(f"router.groups: {self.keep} groups kept out of {self.count}")


@dataclass(frozen=True)
class RouterConfig:
    experts: int
    top: int
    groups: Optional[GroupsConfig] = None

    def __post_init__(self) -> None:
        if not 1 <= self.top <= self.experts:
            raise ConfigError(f"router: {self.top} experts a token out of {self.experts}")
        if self.groups is not None:
            if self.experts % self.groups.count != 0:
                raise ConfigError(f"router: {self.experts} experts do not divide into {self.groups.count} groups")
            if self.top > self.groups.keep * (self.experts // self.groups.count):
                raise ConfigError(f"router: {self.groups.keep} of {self.groups.count} groups do not hold {self.top} experts")


@dataclass(frozen=True)
class ExpertConfig:
    ff: int

    def __post_init__(self) -> None:
        if self.ff < 1:
            raise ConfigError("an expert's ff must be positive")


@dataclass(frozen=True)
class FeedForwardConfig:
    """`kind` "dense": `ff`.  `kind` "moe": `router` and `expert`."""

    kind: str
    ff: Optional[int] = None
    router: Optional[RouterConfig] = None
    expert: Optional[ExpertConfig] = None

    def __post_init__(self) -> None:
        if self.kind == "dense":
            if self.ff is None or self.ff < 1:
                raise ConfigError("a dense mlp needs a positive ff")
            if self.router is not None or self.expert is not None:
                raise ConfigError("a dense mlp has no router and no experts")
        elif self.kind == "moe":
            if self.router is None or self.expert is None:
                raise ConfigError("an mlp of kind 'moe' needs router and expert")
            if self.ff is not None:
                raise ConfigError("an mlp of kind 'moe' has its size under expert")
        else:
            raise ConfigError(f"mlp.kind {self.kind!r}: 'dense' and 'moe' are known")


MIXER_CONFIGS = {"latent_attention": LatentAttentionConfig, "attention": AttentionConfig}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any
    mlp: Optional[FeedForwardConfig] = None

    def __post_init__(self) -> None:
        self.mixer_config()  # reject what does not fit now, by key

    def kind(self) -> str:
        return re.sub(r"_\d+$", "", self.type)  # a numeric suffix marks another set of sizes of the same mixer

    def mixer_config(self):
        kind = self.kind()
        if kind not in MIXER_CONFIGS:
            raise ConfigError(f"layer type {self.type!r}: known mixers are {', '.join(sorted(MIXER_CONFIGS))}")
        if not isinstance(self.mixer, Mapping):
            raise ConfigError(f"the sizes of mixer {self.type!r} must be an object")
        return from_dict(MIXER_CONFIGS[kind], self.mixer, path="mixer")


@dataclass(frozen=True)
class SorovikConfig:
    architecture: str
    vocab: int
    width: int
    norm: NormConfig
    layers: List[LayerConfig]
    max_positions: Optional[int] = None  # not a key of the design: only cache sizing reads it when given

    def __post_init__(self) -> None:
        if self.vocab < 1 or self.width < 1:
            raise ConfigError("vocab and width must be positive")
        if not self.layers:
            raise ConfigError("a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            m = layer.mixer_config()
            j = getattr(m, "kv_from", None)
            if j is None:
                continue
            if not 0 <= j < i or self.layers[j].kind() != "latent_attention":
                raise ConfigError(f"layer {i}: kv_from {j} must name an earlier layer of latent attention")
            source = self.layers[j].mixer_config()
            if source.kv_from is not None:
                raise ConfigError(f"layer {i}: kv_from {j} names a layer without a latent of its own")
            if (source.kv_rank, source.rot_dim, source.rot) != (m.kv_rank, m.rot_dim, m.rot):
                raise ConfigError(f"layer {i} reads layer {j}'s rows: their kv_rank, rot_dim and rotation must be equal")
