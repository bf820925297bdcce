"""Linear attention with a data-dependent decay and a bonus for the current token, on inputs that are blended with the
previous token's (the RWKV time mixing), with a per-request state."""

from __future__ import annotations

from typing import Any, Dict, Mapping, Optional

import torch

from .. import ops
from .base import Mixer, Runtime, StateSpec, TensorSpec, register_part
from .linear import LinearWeights


class WKV(Mixer):
    """Five blends m_s = x_t + (x_(t-1) - x_t) * mu_s of neighbouring tokens (x_(-1) = 0) feed r, k, v (heads x head_dim
    each), the output gate and the decay:
        r = W_r m_r,  k = W_k m_k,  v = W_v m_v,  g = W_g m_g,  alpha = exp(-exp(W_w2 tanh(W_w1 m_w) + w_0))
        o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,      S_t = diag(alpha_t) S_(t-1) + k_t v_t^T       per head
    with S zero at a request's start; then out = W_o (o / rms(o per head) * weight * silu(g)).  The low rank of the decay is
    whatever the folder's w1 and w2 have (random weights are drawn with `DRAWN_RANK`).  The decay from the first
    product's sums on, the state, the bonus, the result's norm and its gate are float32 whatever the activation type.

    A request's state is one float32 row: S in the walking kernel's own layout (`ops.gla_state_elems`), then the last x.
    `names`: local names of the tensors for the roles mu_r, mu_k, mu_v, mu_g, mu_w, r, k, v, g, o, w1, w2, w0, u, norm."""

    replayable = True
    DEFAULT_NAMES = {
        **{f"mu_{s}": f"mu.{s}" for s in "rkvgw"}, **{s: s for s in ("r", "k", "v", "g", "o", "w1", "w2", "w0", "u", "norm")},
    }
    DRAWN_RANK = 64

    def __init__(self, dim: int, heads: int, head_dim: int, eps: float, names: Optional[Mapping[str, str]] = None) -> None:
        if min(heads, head_dim) < 1 or head_dim > ops.MAX_GLA_DIM:
            raise ValueError(f"{heads} heads of {head_dim}: the walking kernel takes 1..{ops.MAX_GLA_DIM} rows")
        self.dim, self.heads, self.head_dim, self.eps = dim, heads, head_dim, float(eps)
        self.names = {**self.DEFAULT_NAMES, **dict(names or {})}
        self.inner = heads * head_dim
        self.matrix_elems = -(-ops.gla_state_elems(heads, head_dim, head_dim) // 4) * 4

    def cache_spec(self) -> StateSpec:
        return StateSpec((-(-(self.matrix_elems + self.dim) // 4) * 4,), torch.float32)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        n = self.names
        specs = {n[f"mu_{s}"]: TensorSpec((self.dim,), precision="stored") for s in "rkvgw"}
        specs.update({n[s]: TensorSpec((self.inner, self.dim)) for s in "rkvg"})
        specs.update({
            n["w1"]: TensorSpec((-self.DRAWN_RANK, self.dim)),
            n["w2"]: TensorSpec((self.inner, -self.DRAWN_RANK)),
            n["w0"]: TensorSpec((self.inner,), precision="stored"),
            n["u"]: TensorSpec((self.heads, self.head_dim), precision="stored"),
            n["norm"]: TensorSpec((self.inner,), init="norm", precision="stored"),
            n["o"]: TensorSpec((self.dim, self.inner)),
        })
        return specs

    def bind(self, tensors: Mapping[str, torch.Tensor], runtime: Runtime) -> None:
        super().bind(tensors, runtime)
        n = self.names
        if tensors[n["w1"]].shape[0] != tensors[n["w2"]].shape[1]:
            raise ValueError(f"the decay's two projections do not meet: {tuple(tensors[n['w1']].shape)} and {tuple(tensors[n['w2']].shape)}")
        self.mu = torch.stack([tensors[n[f"mu_{s}"]].float() for s in "rkvgw"]).contiguous()
        # one matrix whose rows meet five inputs: a decode step's product; the others take its rows apart
        self.joined = LinearWeights.joined([tensors[n[s]] for s in ("r", "k", "v", "g", "w1")], [None] * 5, stream_copy=runtime.stream_copies)
        self.proj = [self.joined.rows(i * self.inner, (i + 1) * self.inner) for i in range(4)]
        self.decay_down = self.joined.rows(4 * self.inner, self.joined.weight.shape[0])
        self.decay_up = LinearWeights(tensors[n["w2"]], tensors[n["w0"]].float())
        self.bonus = tensors[n["u"]].float().reshape(-1).contiguous()
        self.weight = tensors[n["norm"]].float().contiguous()
        self.w_out = LinearWeights(tensors[n["o"]], stream_copy=runtime.stream_copies)

    def forward(self, x: torch.Tensor, batch: Any, cache: Any, write_cache: bool = True) -> torch.Tensor:
        if not write_cache:
            raise ValueError("this mixer cannot read another layer's state")
        mixes = ops.token_mixes(x, self.mu, cache.state, self.matrix_elems, batch)
        if max(batch.q_lens) == 1 and self.decay_down.weight.shape[0] <= self.inner and ops.linear_inputs_takes(mixes, self.joined.weight, self.inner):
            # a decode step: one product for the five inputs, one kernel from its sums to the gated result
            sums = ops.linear_inputs(mixes, self.joined.weight, self.inner, streamed=self.joined.streamed)
            y = ops.wkv_token(
                sums, self.decay_up.weight, self.decay_up.bias, self.bonus, self.weight, cache.state, batch, self.heads, self.head_dim, self.eps, x.dtype,
            )
            return self.w_out(y, partials_ok=True)
        r, k, v, g = (weights(mix) for weights, mix in zip(self.proj, mixes))
        low = ops.act_rows(self.decay_down(mixes[4], out_dtype=torch.float32, partials_ok=True), "tanh", torch.float32)
        logits = ops.gemm_f32(low, self.decay_up.weight, self.decay_up.bias, torch.float32)
        y = ops.wkv(r, k, v, g, logits, self.bonus, self.weight, cache.state, batch, self.heads, self.head_dim, self.head_dim, self.eps)
        return self.w_out(y, partials_ok=True)


register_part("mixer", "wkv", WKV)
