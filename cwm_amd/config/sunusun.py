"""Typed configuration of the Sunusun decoder.

config.json names the vocabulary, the width, one eps for every norm, a factor on the logits and a list of layers.  Every
layer names its mixer (`type`: "parallel" or "wkv"), the mixer's sizes (`mixer`) and its feed-forward (`mlp`, null for
none).  `weights_of` makes a layer run on the tensors of another one, whose mixer and feed-forward it must repeat; caches
and states are not shared.  Strict as every configuration: an unknown key is an error that names it.
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
class TemperatureConfig:
    """A query at position p is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1)."""

    coef: float
    every: int

    def __post_init__(self) -> None:
        if self.every < 1:
            raise ConfigError("q_temp.every must be at least 1")


@dataclass(frozen=True)
class AttentionConfig:
    """`heads` query heads on `kv_heads` key/value heads; queries and keys of `dim`, values of `vdim` per head."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[TemperatureConfig] = None

    def __post_init__(self) -> None:
        if min(self.heads, self.kv_heads, self.dim, self.vdim) < 1:
            raise ConfigError("an attention mixer's sizes must be positive")
        if self.heads % self.kv_heads != 0:
            raise ConfigError(f"{self.heads} query heads do not divide into {self.kv_heads} key/value heads")
        if self.scale <= 0:
            raise ConfigError("scale must be positive")


@dataclass(frozen=True)
class RecurrenceConfig:
    width: int  # elements of the gated recurrence's state

    def __post_init__(self) -> None:
        if self.width < 1:
            raise ConfigError("the recurrence's width must be positive")


@dataclass(frozen=True)
class ParallelConfig:
    """An attention (`left`) and a gated recurrence (`right`) side by side."""

    left: AttentionConfig
    right: RecurrenceConfig


@dataclass(frozen=True)
class WKVConfig:
    heads: int
    dim: int  # rows and columns of a head's state

    def __post_init__(self) -> None:
        if min(self.heads, self.dim) < 1:
            raise ConfigError("a wkv mixer's sizes must be positive")


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str
    ff: int

    def __post_init__(self) -> None:
        if self.kind != "dense":
            raise ConfigError(f"mlp.kind {self.kind!r}: 'dense' is known")
        if self.ff < 1:
            raise ConfigError("a dense mlp needs a positive ff")


MIXER_CONFIGS = {"parallel": ParallelConfig, "wkv": WKVConfig}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any
    mlp: Optional[FeedForwardConfig] = None
    weights_of: Optional[int] = None

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
class SunusunConfig:
    architecture: str
    vocab: int
    width: int
    norm: NormConfig
    layers: List[LayerConfig]
    logit_scale: float = 1.0
    max_positions: Optional[int] = None  # not a key of the design: only cache sizing reads it when given

    def __post_init__(self) -> None:
        if self.vocab < 1 or self.width < 1:
            raise ConfigError("vocab and width must be positive")
        if not self.layers:
            raise ConfigError("a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            if layer.weights_of is None:
                continue
            if not 0 <= layer.weights_of < len(self.layers):
                raise ConfigError(f"layer {i}: weights_of {layer.weights_of} names no layer")
            other = self.layers[layer.weights_of]
            if (layer.kind(), layer.mixer_config(), layer.mlp) != (other.kind(), other.mixer_config(), other.mlp):
                raise ConfigError(f"layer {i} uses layer {layer.weights_of}'s tensors: their mixers and feed-forwards must be equal")
            self.owner(i)

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses (i itself, or where its `weights_of` leads)."""
        seen = [i]
        while self.layers[seen[-1]].weights_of is not None:
            j = self.layers[seen[-1]].weights_of
            if j in seen:
                raise ConfigError(f"layer {i}: weights_of leads in a circle ({' -> '.join(map(str, seen + [j]))})")
            seen.append(j)
        return seen[-1]
