"""Entry points of the kernels between a mixer's projections and its attention: rows of attention through a cached latent
(`csrc/latent_rows.hip`), and queries and keys that pass a short convolution (`csrc/conv_qk.hip`).  Shapes, types and
devices are checked on the host; there is no CPU path."""

from __future__ import annotations

import ctypes
from typing import Any, Optional, Tuple

import torch

from . import build as _build

MAX_CONV_QK_TAPS = 16  # csrc/conv_qk.hip: CONVQK_MAX_TAPS
MAX_CONV_QK_CHANNELS = 60 * 1024 // 4  # csrc/conv_qk.hip: CONVQK_MAX_LDS


def _base():
    from . import KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream  # the shared helpers of this package

    return KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream


def _source(x: torch.Tensor, width: int, what: str) -> Tuple[int, int, int, int]:
    """(rows, distance of rows, number of partial sums, their distance) of a projection with at least `width` columns."""
    KernelError = _base()[0]
    if x.dim() == 3 and x.dtype == torch.float32 and x.stride(2) == 1:
        rows, stride, parts, part_stride = x.shape[1], x.stride(1), x.shape[0], x.stride(0)
    elif x.dim() == 2 and x.stride(1) == 1:
        rows, stride, parts, part_stride = x.shape[0], (x.stride(0) if x.shape[0] > 1 else x.shape[1]), 1, 0
    else:
        raise KernelError(f"{what} must be [T, N] with contiguous rows or float32 partial sums [P, T, N]")
    if x.shape[-1] < width:
        raise KernelError(f"{what} has {x.shape[-1]} columns, {width} are needed")
    return rows, stride, parts, part_stride


def _paged(cache: torch.Tensor, block_table: torch.Tensor, n_kv: int, head_dim: int, dtype: torch.dtype) -> Tuple[int, int, int]:
    """(pages, page size, table width) of a paged cache after checking it."""
    KernelError, _, _, _i32, *_ = _base()
    if cache.dim() != 4 or cache.shape[1] != 2 or cache.shape[2] != n_kv or cache.shape[3] % head_dim != 0 or not cache.is_contiguous():
        raise KernelError(f"cache {tuple(cache.shape)} does not fit {n_kv} heads of size {head_dim}")
    if cache.dtype != dtype:
        raise KernelError("the cache and the queries must have one type")
    _i32(block_table, "block_table")
    if block_table.dim() != 2:
        raise KernelError("block_table must be [B, W]")
    return cache.shape[0], cache.shape[3] // head_dim, block_table.shape[1]


def latent_rows(
    q_src: torch.Tensor, kv_src: Optional[torch.Tensor], n_heads: int, lead: int, n_rest: int, rank: int, row: int,
    weight: Optional[torch.Tensor], eps: float, batch: Any, inv_freq: Optional[torch.Tensor], out_dtype: torch.dtype,
    cache: Optional[torch.Tensor] = None, block_table: Optional[torch.Tensor] = None,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """`q_src` [T, >= n_heads * (lead + n_rest)] with a head's rotated part first, `kv_src` [T, >= lead + rank] with the
    shared rotated part first (either may be float32 partial sums [P, T, ...], added in order; both of one type; `kv_src`
    None where another layer has written the cache).  The latent is divided by its root mean square and multiplied by
    `weight` (float32 [rank]); rotated parts turn by positions * inv_freq (float32 [lead / 2], adjacent pairs); the row
    [rotated | latent | zeros up to `row`] goes into the paged `cache` as the token's key and as its value.  Returns `ask`
    [T, n_heads, row] in `out_dtype` with the leading `lead` elements of every head filled in, and the heads' unrotated
    parts as [T, n_heads, n_rest] (a view of `q_src` where that has the right type already)."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(q_src, kv_src, weight, inv_freq, cache, block_table)
    n_tokens, q_stride, q_parts, q_part_stride = _source(q_src, n_heads * (lead + n_rest), "the queries' projection")
    if n_tokens != batch.n_tokens:
        raise KernelError(f"the projection has {n_tokens} rows, the step {batch.n_tokens} tokens")
    kv_stride = kv_part_stride = 0
    kv_parts = 1
    num_pages = page_size = table_width = 0
    if kv_src is not None:
        kv_rows, kv_stride, kv_parts, kv_part_stride = _source(kv_src, lead + rank, "the latent's projection")
        if kv_rows != n_tokens or kv_src.dtype != q_src.dtype:
            raise KernelError("both projections must have one type and one number of rows")
        if cache is None or block_table is None or weight is None:
            raise KernelError("a cached row needs its norm's weight, a cache and a block table")
        if weight.dtype != torch.float32 or weight.shape != (rank,) or not weight.is_contiguous():
            raise KernelError(f"the latent's norm weight must be a contiguous float32 [{rank}] tensor")
        num_pages, page_size, table_width = _paged(cache, block_table, 1, row, out_dtype)
    if inv_freq is not None and (inv_freq.dtype != torch.float32 or inv_freq.numel() < lead // 2 or not inv_freq.is_contiguous()):
        raise KernelError(f"the rotary table must hold {lead // 2} contiguous float32 values")
    ask = torch.empty((n_tokens, n_heads, row), dtype=out_dtype, device=q_src.device)
    view = q_src.dim() == 2 and q_src.dtype == out_dtype
    rest = None if view else torch.empty((n_tokens, n_heads, n_rest), dtype=out_dtype, device=q_src.device)
    lib = _build.load("latent_rows")
    _check(
        lib,
        lib.cwm_latent_rows(
            _ptr(q_src), ctypes.c_long(q_stride), ctypes.c_int(q_parts), ctypes.c_long(q_part_stride), _ptr(kv_src), ctypes.c_long(kv_stride),
            ctypes.c_int(kv_parts), ctypes.c_long(kv_part_stride), ctypes.c_int(_code(q_src.dtype)), _ptr(weight), ctypes.c_float(eps),
            _ptr(batch.positions), _ptr(batch.seq_of_token), _ptr(inv_freq), _ptr(ask), _ptr(rest), ctypes.c_int(_code(out_dtype)), _ptr(cache),
            _ptr(block_table), ctypes.c_int(table_width), ctypes.c_int(page_size), ctypes.c_int(num_pages), ctypes.c_int(n_tokens),
            ctypes.c_int(n_heads), ctypes.c_int(lead), ctypes.c_int(n_rest), ctypes.c_int(rank), ctypes.c_int(row), _stream(),
        ),
    )
    if view:
        width = lead + n_rest
        rest = q_src[:, : n_heads * width].unflatten(1, (n_heads, width))[:, :, lead:]
    return ask, rest


def conv_qk_rope_write(
    proj: torch.Tensor, n_q_heads: int, n_kv_heads: int, dim: int, head_dim: int, bias: Optional[torch.Tensor], by_tap: torch.Tensor,
    q_weight: Optional[torch.Tensor], k_weight: Optional[torch.Tensor], eps: float, batch: Any, inv_freq: Optional[torch.Tensor],
    out_dtype: torch.dtype, cache: torch.Tensor, block_table: torch.Tensor, state: Optional[torch.Tensor], gate: bool = False,
) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """From the joined projection `proj` ([T, (Hq + Hkv) * dim (+ Hq gates)], or float32 partial sums [P, T, ...] of it):
    queries and keys plus `bias` (float32, a value a channel, or None) pass a causal convolution over their sequence,
    channel by channel (`by_tap` float32 [taps, channels], the last row the current token's; a sequence's last taps - 1
    inputs live in its row of `state`, float32 [slots, >= (taps - 1) * channels], read by the portion's first tokens and
    then replaced).  The key heads as they then are become the values; queries and keys are each divided by the root mean
    square of their whole projection and multiplied by `q_weight` / `k_weight` (float32, one value an element; None: no
    norm), rotated by positions * inv_freq (float32 [head_dim / 2], adjacent pairs), and keys and values go into the
    paged `cache`.  Returns the queries [T, Hq, head_dim] in `out_dtype` (zeros from `dim` on) and, with `gate`, the
    sigmoid of the gates (float32 [T, Hq])."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(proj, bias, by_tap, q_weight, k_weight, inv_freq, cache, block_table, state)
    channels = (n_q_heads + n_kv_heads) * dim
    n_tokens, stride, parts, part_stride = _source(proj, channels + (n_q_heads if gate else 0), "the projection")
    if n_tokens != batch.n_tokens:
        raise KernelError(f"the projection has {n_tokens} rows, the step {batch.n_tokens} tokens")
    if channels > MAX_CONV_QK_CHANNELS:
        raise KernelError(f"{channels} channels of queries and keys: the kernel takes up to {MAX_CONV_QK_CHANNELS}")
    taps = by_tap.shape[0]
    vectors = (("bias", bias, (channels,)), ("the convolution's weight", by_tap, (taps, channels)), ("the queries' norm weight", q_weight, (n_q_heads * dim,)),
               ("the keys' norm weight", k_weight, (n_kv_heads * dim,)), ("the rotary table", inv_freq, (head_dim // 2,)))
    for what, t, shape in vectors:
        if t is not None and (t.dtype != torch.float32 or tuple(t.shape) != shape or not t.is_contiguous()):
            raise KernelError(f"{what} must be a contiguous float32 {list(shape)} tensor")
    if not 1 <= taps <= MAX_CONV_QK_TAPS:
        raise KernelError(f"{taps} taps are outside 1..{MAX_CONV_QK_TAPS}")
    if taps > 1 and (state is None or state.dtype != torch.float32 or state.dim() != 2 or state.shape[1] < (taps - 1) * channels or not state.is_contiguous()):
        raise KernelError(f"the state must be a contiguous float32 [slots, >= {(taps - 1) * channels}] tensor")
    num_pages, page_size, table_width = _paged(cache, block_table, n_kv_heads, head_dim, out_dtype)
    q = torch.empty((n_tokens, n_q_heads, head_dim), dtype=out_dtype, device=proj.device)
    gates = torch.empty((n_tokens, n_q_heads), dtype=torch.float32, device=proj.device) if gate else None
    # a step of single tokens (a decode step) moves the state in the same launch: a token's block is its only reader
    q_lens = getattr(batch, "q_lens", None)
    mode = 2 if q_lens and max(q_lens) == 1 else 1
    carried = state if taps > 1 else None
    lib = _build.load("conv_qk")
    _check(
        lib,
        lib.cwm_conv_qk(
            _ptr(proj), ctypes.c_int(_code(proj.dtype)), ctypes.c_long(stride), ctypes.c_int(parts), ctypes.c_long(part_stride), _ptr(bias),
            _ptr(by_tap), ctypes.c_int(taps), _ptr(carried), ctypes.c_long(carried.shape[1] if carried is not None else 0), _ptr(batch.state_slots),
            _ptr(batch.cu_q), _ptr(batch.seq_of_token), ctypes.c_int(carried.shape[0] if carried is not None else 0), ctypes.c_int(batch.n_seqs),
            ctypes.c_int(mode), _ptr(q), ctypes.c_int(_code(out_dtype)), _ptr(gates), _ptr(q_weight), _ptr(k_weight), ctypes.c_float(eps),
            _ptr(batch.positions), _ptr(inv_freq), _ptr(cache), _ptr(block_table), ctypes.c_int(table_width), ctypes.c_int(page_size),
            ctypes.c_int(num_pages), ctypes.c_int(n_tokens), ctypes.c_int(n_q_heads), ctypes.c_int(n_kv_heads), ctypes.c_int(dim),
            ctypes.c_int(head_dim), _stream(),
        ),
    )
    return q, gates
