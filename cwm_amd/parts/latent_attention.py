"""Causal attention whose keys and values are rebuilt from one cached latent row per token."""

from __future__ import annotations

from typing import Any, Dict, Mapping, Optional

import torch

from .. import ops
from .attention import MAX_HEAD_DIM
from .base import Mixer, PagedKVSpec, PartChoice, PositionEncoding, Runtime, TensorSpec, register_part
from .linear import LinearWeights


class LatentAttention(Mixer):
    """Keys and values through a latent: W_dkv s = [c | kr], c <- rms(c) w_kv; head h has the key [W_uk,h c | rot(kr)] and
    the value W_uv,h c.  Queries q_h = [n_h | r_h] with `head_dim` unrotated and `rot_dim` rotated elements are W_q s, or
    with `q_rank` come through a latent of their own: cq = rms(W_dq s) w_q, q_h = (W_uq cq)_h.  Scores scale * q.k over the
    `window` keys up to the query's own (None: the causal past), softmax (with `sink` its denominator also holds
    exp(sink_h), a stored number per head that has no key and no value and is not scaled); the heads' results, times
    sigmoid(W_g s) element by element where `gate`, go through W_o.

    Only [rot(kr) | c] is cached, one row a token, and attention runs on those rows directly: since
    n_h . (W_uk,h c) = (W_uk,h^T n_h) . c, head h asks with [rot(r_h) | W_uk,h^T n_h], all heads read the one
    row as key and as value, and W_uv,h is applied to the weighted sum of latents afterwards.  That is
    attention with one key/value head of size rot_dim + kv_rank (rounded up to a multiple of 16 with zeros), which the
    paged attention kernels serve; the rotated part leads the row so that the rotation's pairs start at an even element.
    The position encoding turns the first elements of the rotated part (its table may be shorter than rot_dim / 2: the
    rest of the part passes unchanged), in adjacent pairs or in halves of the turned elements.

    With `own_kv=False` the mixer has no W_dkv: it is run on the rows that another layer of equal kv_rank, rot_dim and
    rotation has cached in the same step (`write_cache` false), with queries, W_uk, W_uv, window and sink of its own.
    `cache_window` is what the cache keeps (default: `window`): a layer whose rows another layer reads through a longer
    window keeps that longer one."""

    _KEEP_WINDOW = object()

    def __init__(
        self, dim: int, n_heads: int, head_dim: int, rot_dim: int, v_dim: int, kv_rank: int, q_rank: Optional[int], scale: float, eps: float,
        position_encoding: Optional[PartChoice] = None, window: Optional[int] = None, cache_window: Any = _KEEP_WINDOW, sink: bool = False,
        gate: bool = True, own_kv: bool = True,
    ) -> None:
        self.row = -(-(rot_dim + kv_rank) // 16) * 16  # a cached row, and the size of the one key/value head
        if self.row > MAX_HEAD_DIM:
            raise ValueError(f"a cached row of {rot_dim} + {kv_rank} elements is more than the {MAX_HEAD_DIM} the attention kernels take")
        if rot_dim % 2 != 0:
            raise ValueError("the rotated part needs an even size")
        if window is not None and window < 1:
            raise ValueError("a window holds at least the query's own key")
        self.dim, self.n_heads, self.head_dim, self.rot_dim, self.v_dim = dim, n_heads, head_dim, rot_dim, v_dim
        self.kv_rank, self.q_rank, self.scale, self.eps = kv_rank, q_rank, float(scale), float(eps)
        self.window, self.sink, self.gate, self.own_kv = window, sink, gate, own_kv
        self.cache_window = window if cache_window is self._KEEP_WINDOW else cache_window
        if self.cache_window is not None and (window is None or self.cache_window < window):
            raise ValueError("the cache must keep at least the rows of the mixer's own window")
        self.q_norm = None
        if q_rank is not None:
            self.q_norm = PartChoice("group_rmsnorm", {"dim": q_rank, "eps": eps, "groups": 1, "tensor": "dq.norm"}).build("norm")
        self.position_encoding: Optional[PositionEncoding] = (
            position_encoding.build("position_encoding") if position_encoding is not None else None
        )

    @property
    def replayable(self) -> bool:  # type: ignore[override]
        return self.position_encoding is None or self.position_encoding.replayable

    def cache_spec(self) -> PagedKVSpec:
        return PagedKVSpec(n_kv_heads=1, head_dim=self.row, window=self.cache_window)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        h = self.n_heads
        q_out = h * (self.head_dim + self.rot_dim)
        if self.q_rank is None:
            specs = {"q": TensorSpec((q_out, self.dim))}
        else:
            specs = {"dq": TensorSpec((self.q_rank, self.dim)), **self.q_norm.tensor_specs(), "uq": TensorSpec((q_out, self.q_rank))}
        if self.own_kv:
            specs["dkv"] = TensorSpec((self.kv_rank + self.rot_dim, self.dim))
            specs["dkv.norm"] = TensorSpec((self.kv_rank,), init="norm", precision="stored")
        specs["uk"] = TensorSpec((h * self.head_dim, self.kv_rank))
        specs["uv"] = TensorSpec((h * self.v_dim, self.kv_rank))
        if self.sink:
            specs["sink"] = TensorSpec((h,), init="zeros", precision="stored")
        if self.gate:
            specs["g"] = TensorSpec((h * self.v_dim, self.dim))
        specs["o"] = TensorSpec((self.dim, h * self.v_dim))
        return specs

    def bind(self, tensors: Mapping[str, torch.Tensor], runtime: Runtime) -> None:
        super().bind(tensors, runtime)
        h, hd, rd, kr = self.n_heads, self.head_dim, self.rot_dim, self.kv_rank
        device = tensors["uk"].device
        order = torch.arange(rd)
        self.table = None
        if self.position_encoding is not None:
            self.position_encoding.bind({}, runtime)
            table = self.position_encoding.rotary_table()
            if table is not None:
                turned = 2 * table.numel()
                if turned > rd:
                    raise ValueError(f"a rotation of {turned} elements does not fit the rotated part of {rd}")
                if self.position_encoding.rotary_pairing() == "halves":
                    # the kernels turn adjacent elements: bring element i and i + turned / 2 side by side, once, in the rows of
                    # the queries' and the shared key's rotated parts (scores are sums over them, and nothing else reads them)
                    half = turned // 2
                    order = torch.cat([torch.stack([torch.arange(half), torch.arange(half) + half], dim=1).reshape(-1), torch.arange(turned, rd)])
                self.table = torch.zeros(max(1, rd // 2), dtype=torch.float32, device=device)
                self.table[: table.numel()] = table.to(device)
        order = order.to(device)
        q = tensors["q" if self.q_rank is None else "uq"]
        q = q.reshape(h, hd + rd, q.shape[1])
        # rows head by head as [r_h | n_h], so that the rotated part leads here too
        q = torch.cat([q[:, hd:][:, order], q[:, :hd]], dim=1).reshape(h * (hd + rd), q.shape[2])
        # one product for everything that reads s: [kr | c] (the rotated part first, as the cache keeps it), the queries
        # (or the latent they come from), the gate
        down = []
        if self.own_kv:
            dkv = tensors["dkv"]
            down.append(torch.cat([dkv[kr:][order], dkv[:kr]], dim=0))
            self.kv_weight = tensors["dkv.norm"].float().contiguous()
        down.append(q if self.q_rank is None else tensors["dq"])
        if self.gate:
            down.append(tensors["g"])
        self.down = LinearWeights.joined(down, [None] * len(down), stream_copy=runtime.stream_copies)
        if self.q_rank is not None:
            self.q_norm.bind({"dq.norm": tensors["dq.norm"]}, runtime)
            self.up_q = LinearWeights(q, stream_copy=runtime.stream_copies)
        pad = self.row - rd - kr  # zeros at the end of a cached row
        uk = tensors["uk"].reshape(h, hd, kr).transpose(1, 2)  # [h, kv_rank, head_dim]: n_h -> W_uk,h^T n_h
        uv = tensors["uv"].reshape(h, self.v_dim, kr)  # [h, v_dim, kv_rank]: sum of latents -> value
        self.w_uk = torch.cat([uk, uk.new_zeros((h, pad, hd))], dim=1).contiguous()
        self.w_uv = torch.cat([uv, uv.new_zeros((h, self.v_dim, pad))], dim=2).contiguous()
        self.sinks = tensors["sink"].float().contiguous() if self.sink else None
        self.w_o = LinearWeights(tensors["o"], stream_copy=runtime.stream_copies)

    def forward(self, x: torch.Tensor, batch: Any, cache: Any, write_cache: bool = True) -> torch.Tensor:
        if write_cache and not self.own_kv:
            raise ValueError("a mixer without a latent of its own reads another layer's rows")
        h, hd, rd, kr, row = self.n_heads, self.head_dim, self.rot_dim, self.kv_rank, self.row
        kv_width = rd + kr if self.own_kv else 0
        down = self.down(x, partials_ok=self.q_rank is None and not self.gate)  # [T, kv_width + queries (+ gate)]
        if self.q_rank is None:
            q_src = down[..., kv_width : kv_width + h * (hd + rd)]
        else:
            q_src = self.up_q(self.q_norm.forward(down[:, kv_width : kv_width + self.q_rank], None))
        # what each head asks the cached rows with: [r_h | W_uk,h^T n_h]
        ask, rest = ops.latent_rows(
            q_src, down[..., :kv_width] if write_cache else None, h, rd, hd, kr, row, self.kv_weight if write_cache else None, self.eps, batch,
            self.table, self.runtime.act_dtype, cache.cache if write_cache else None, cache.block_table if write_cache else None,
        )
        ops.absorb_queries(rest, ask, rd, self.w_uk)
        mixed = ops.paged_attention(ask, cache.cache, cache.block_table, batch, self.window, self.scale, sink=self.sinks).unflatten(1, (h, row))
        values = ops.expand_values(mixed, rd, self.w_uv)  # [T, h * v_dim]
        if self.gate:
            values = ops.sigmoid_mul(values, down[:, down.shape[1] - h * self.v_dim :])
        return self.w_o(values, partials_ok=True)


register_part("mixer", "latent_attention", LatentAttention)
