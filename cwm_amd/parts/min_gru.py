"""A recurrence over single elements, gated without looking at its own state (minGRU), with a per-request state."""

from __future__ import annotations

from typing import Any, Dict, Mapping, Optional

import torch

from .. import ops
from .base import Mixer, Runtime, StateSpec, TensorSpec, register_part
from .linear import LinearWeights


class MinGRU(Mixer):
    """z = sigmoid(W_z x + b_z), u = W_x x + b_x (`width` values each); element by element
        S_t = (1 - z) S_(t-1) + z g(u),      g(u) = u + 1/2 for u >= 0, sigmoid(u) for u < 0
    with S zero at a request's start; then out = W_o (S_t * silu(W_g x)).  Gates, candidates, state and output gate are
    float32 whatever the activation type.  A request's state is S, float32 [width].  `names`: local names of the tensors
    for the roles z, z_bias, x, x_bias, g and o."""

    replayable = True
    DEFAULT_NAMES = {"z": "z", "z_bias": "z.b", "x": "x", "x_bias": "x.b", "g": "g", "o": "o"}

    def __init__(self, dim: int, width: int, names: Optional[Mapping[str, str]] = None) -> None:
        if min(dim, width) < 1:
            raise ValueError("a gated recurrence needs positive sizes")
        self.dim, self.width = dim, width
        self.names = {**self.DEFAULT_NAMES, **dict(names or {})}

    def cache_spec(self) -> StateSpec:
        return StateSpec((self.width,), torch.float32)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        n = self.names
        return {
            n["z"]: TensorSpec((self.width, self.dim)),
            n["z_bias"]: TensorSpec((self.width,), precision="stored"),
            n["x"]: TensorSpec((self.width, self.dim)),
            n["x_bias"]: TensorSpec((self.width,), precision="stored"),
            n["g"]: TensorSpec((self.width, self.dim)),
            n["o"]: TensorSpec((self.dim, self.width)),
        }

    def bind(self, tensors: Mapping[str, torch.Tensor], runtime: Runtime) -> None:
        super().bind(tensors, runtime)
        n = self.names
        # the biases are added in the recurrence's own kernel, in float32
        self.proj = LinearWeights.joined([tensors[n[r]] for r in ("z", "x", "g")], [None] * 3, stream_copy=runtime.stream_copies)
        self.w_out = LinearWeights(tensors[n["o"]], stream_copy=runtime.stream_copies)
        self.z_bias = tensors[n["z_bias"]].float().contiguous()
        self.x_bias = tensors[n["x_bias"]].float().contiguous()

    def forward(self, x: torch.Tensor, batch: Any, cache: Any, write_cache: bool = True) -> torch.Tensor:
        if not write_cache:
            raise ValueError("a gated recurrence cannot read another layer's state")
        y = ops.min_gru(self.proj(x, partials_ok=True), self.z_bias, self.x_bias, cache.state, batch, self.runtime.act_dtype)
        return self.w_out(y, partials_ok=True)


register_part("mixer", "min_gru", MinGRU)
