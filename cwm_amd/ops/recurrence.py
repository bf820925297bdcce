"""Entry points of the kernels of layers with a gated element-wise recurrence, of blends of a token with the one before
it, of linear attention with a bonus for the current token, and of results that are normalised before they join the
residual (`csrc/min_gru.hip`, `csrc/token_mix.hip`, `csrc/linear_attention.hip`, `csrc/normed_sum.hip`), and of an
embedding with sinusoidal positions (`csrc/rowwise.hip`).  Shapes, types and devices are checked on the host; there is
no CPU path."""

from __future__ import annotations

import ctypes
from typing import Any, Optional, Sequence, Tuple

import torch

from . import build as _build
from .sequence import step_segments
from .streams import RoutedSum

MAX_TOKEN_MIXES = 8  # csrc/token_mix.hip: TMIX_MAX
MAX_NORMED_ADDENDS = 4  # csrc/normed_sum.hip: NSUM_MAX
MIN_GRU_WALK = 32  # tokens of the longest portion that a step still walks as a whole; longer ones go in segments
MIN_GRU_SEGMENT = 16  # tokens of a segment at least
MIN_GRU_SEGMENTS = 128  # and segments of a portion at most


def _base():
    from . import KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream  # the shared helpers of this package

    return KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream


def embedding_sinusoid(tokens: torch.Tensor, table: torch.Tensor, positions: torch.Tensor, turns: torch.Tensor, scale: float = 1.0) -> torch.Tensor:
    """float32 [T, D]: `scale` times the rows of `table` ([V, D]) for int32 `tokens`, plus the sinusoidal vector of
    int32 `positions`: entry 2i is sin(p f_i), entry 2i + 1 cos(p f_i), with `turns` float64 [ceil(D / 2)] holding
    f_i / (2 pi)."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(tokens, table, positions, turns)
    _i32(tokens, "tokens")
    _i32(positions, "positions")
    if table.dim() != 2 or not table.is_contiguous():
        raise KernelError("embedding table must be a contiguous [V, D] tensor")
    n, dim = tokens.numel(), table.shape[1]
    if positions.numel() != n:
        raise KernelError("one position per token is needed")
    if turns.dtype != torch.float64 or turns.shape != ((dim + 1) // 2,) or not turns.is_contiguous():
        raise KernelError(f"the positions' frequencies must be float64 [{(dim + 1) // 2}]")
    lib = _build.load("rowwise")
    out = torch.empty((n, dim), dtype=torch.float32, device=table.device)
    _check(
        lib,
        lib.cwm_embedding_sinusoid(
            _ptr(out), _ptr(table), ctypes.c_int(_code(table.dtype)), _ptr(tokens), _ptr(positions), _ptr(turns), ctypes.c_int(n),
            ctypes.c_int(dim), ctypes.c_int(table.shape[0]), ctypes.c_float(scale), _stream(),
        ),
    )
    return out


class NormedSum:
    """A sum that has not been done yet: `terms` is a list of (tensor, weight, factor), each tensor ([T, D], rows may lie
    apart, float32 partial sums [P, T, D], or a `RoutedSum`) divided by its rows' root mean square (`eps` inside the root) and multiplied
    by its weight (float32 [D]) and its factor.  The norm that reads the residual next adds the terms up in their order,
    in float32 (`add_normed_rmsnorm`)."""

    def __init__(self, terms, eps: float) -> None:
        self.terms = [(t, w, float(c)) for t, w, c in terms]
        self.eps = float(eps)


def _addends(terms: Sequence[Tuple[Any, float]], n_tokens: int, dim: int):
    """ctypes arrays (pointers, types, row distances, numbers of partial sums or of rows in a weighted sum, the partial sums'
    distances, factors, and for weighted sums the rows' places and weights) of addends."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    n = len(terms)
    ptrs, dtypes, lds, partials = (ctypes.c_void_p * n)(), (ctypes.c_int * n)(), (ctypes.c_long * n)(), (ctypes.c_int * n)()
    strides, scales = (ctypes.c_long * n)(), (ctypes.c_float * n)()
    row_index, row_weight = (ctypes.c_void_p * n)(), (ctypes.c_void_p * n)()
    for i, (t, c) in enumerate(terms):
        if isinstance(t, RoutedSum):
            top = t.groups.top
            _need_gpu(t.rows, t.weights, t.groups.pair_row)
            if t.rows.dtype != torch.float32 or t.rows.dim() != 2 or t.rows.shape[1] != dim or not t.rows.is_contiguous():
                raise KernelError(f"the experts' rows must be a contiguous float32 [rows, {dim}] tensor")
            if t.weights.dtype != torch.float32 or tuple(t.weights.shape) != (n_tokens, top) or not t.weights.is_contiguous():
                raise KernelError(f"the weights of a weighted sum must be float32 [{n_tokens}, {top}]")
            if t.groups.pair_row.numel() != n_tokens * top:
                raise KernelError("the list of rows does not fit the tokens")
            ptrs[i], dtypes[i], scales[i], lds[i], partials[i] = t.rows.data_ptr(), _code(torch.float32), c, dim, top
            row_index[i], row_weight[i] = t.groups.pair_row.data_ptr(), t.weights.data_ptr()
            continue
        _need_gpu(t)
        if t.dim() == 3:
            if t.dtype != torch.float32 or not t.is_contiguous() or tuple(t.shape[1:]) != (n_tokens, dim):
                raise KernelError(f"partial sums {tuple(t.shape)} must be contiguous float32 [P, {n_tokens}, {dim}]")
            partials[i], strides[i], lds[i] = t.shape[0], n_tokens * dim, dim
        else:
            if t.dim() != 2 or t.stride(1) != 1 or tuple(t.shape) != (n_tokens, dim):
                raise KernelError(f"an addend {tuple(t.shape)} does not match the residual stream [{n_tokens}, {dim}]")
            partials[i], strides[i], lds[i] = 1, 0, (t.stride(0) if n_tokens > 1 else dim)
        ptrs[i], dtypes[i], scales[i] = t.data_ptr(), _code(t.dtype), c
    return ptrs, dtypes, lds, partials, strides, scales, row_index, row_weight


def add_normed_rmsnorm(
    h: torch.Tensor, delta: NormedSum, weight: torch.Tensor, eps: float, out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """`h` (float32 [T, D]) += `delta` in place, then h / sqrt(mean(h^2) + eps) * weight (float32 [D]) in `out_dtype`.
    With `rows` (int32 [R]) only those rows are normalised and `h` is not changed (the sum with `delta` is still what is
    normalised)."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(h, weight, rows)
    if h.dtype != torch.float32 or h.dim() != 2 or not h.is_contiguous():
        raise KernelError("the residual stream must be a contiguous float32 [T, D] tensor")
    n_tokens, dim = h.shape
    if not 1 <= len(delta.terms) <= MAX_NORMED_ADDENDS:
        raise KernelError(f"{len(delta.terms)} addends: the kernel takes 1..{MAX_NORMED_ADDENDS}")
    for what, t in [("the norm's weight", weight)] + [("an addend's weight", w) for _, w, _ in delta.terms]:
        _need_gpu(t)
        if t.dtype != torch.float32 or t.shape != (dim,) or not t.is_contiguous():
            raise KernelError(f"{what} must be a contiguous float32 [{dim}] tensor")
    if rows is not None:
        _i32(rows, "rows")
    ptrs, dtypes, lds, partials, strides, scales, row_index, row_weight = _addends([(t, c) for t, _, c in delta.terms], n_tokens, dim)
    weights = (ctypes.c_void_p * len(delta.terms))(*[w.data_ptr() for _, w, _ in delta.terms])
    n_out = n_tokens if rows is None else rows.numel()
    out = torch.empty((n_out, dim), dtype=out_dtype, device=h.device)
    lib = _build.load("normed_sum")
    _check(
        lib,
        lib.cwm_normed_sum(
            _ptr(h), ctypes.c_int(len(delta.terms)), ptrs, dtypes, lds, partials, strides, scales, weights, row_index, row_weight, ctypes.c_float(delta.eps),
            _ptr(weight), ctypes.c_float(eps), _ptr(out), ctypes.c_int(_code(out_dtype)), _ptr(rows), ctypes.c_int(n_out), ctypes.c_int(dim), _stream(),
        ),
    )
    return out


def token_mixes(x: torch.Tensor, mu: torch.Tensor, state: torch.Tensor, state_offset: int, batch: Any) -> torch.Tensor:
    """[n, T, D] in the type of `x`: x_t + (x_(t-1) - x_t) * mu_s for every row mu_s of `mu` (float32 [n, D]) over the
    step's tokens `x` (contiguous [T, D]); the row before a portion's first token lies in the sequence's row of `state`
    (float32 [slots, m], `D` values from `state_offset` on, zeros when a request is admitted), which then receives the
    portion's last row."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(x, mu, state)
    if x.dim() != 2 or not x.is_contiguous() or x.shape[0] != batch.n_tokens:
        raise KernelError(f"x must be a contiguous [{batch.n_tokens}, D] tensor")
    n_tokens, dim = x.shape
    if mu.dtype != torch.float32 or mu.dim() != 2 or mu.shape[1] != dim or not mu.is_contiguous() or not 1 <= mu.shape[0] <= MAX_TOKEN_MIXES:
        raise KernelError(f"the blends' weights must be a contiguous float32 [1..{MAX_TOKEN_MIXES}, {dim}] tensor")
    if state.dtype != torch.float32 or state.dim() != 2 or not state.is_contiguous() or not 0 <= state_offset <= state.shape[1] - dim:
        raise KernelError(f"the state must be a contiguous float32 [slots, n] tensor with {dim} values from {state_offset} on")
    out = torch.empty((mu.shape[0], n_tokens, dim), dtype=x.dtype, device=x.device)
    lib = _build.load("token_mix")
    _check(
        lib,
        lib.cwm_token_mix(
            _ptr(x), ctypes.c_int(_code(x.dtype)), _ptr(mu), ctypes.c_int(mu.shape[0]), _ptr(out), ctypes.c_long(n_tokens * dim),
            _ptr(state), ctypes.c_long(state.shape[1]), ctypes.c_long(state_offset), _ptr(batch.state_slots), _ptr(batch.cu_q),
            _ptr(batch.seq_of_token), ctypes.c_int(state.shape[0]), ctypes.c_int(n_tokens), ctypes.c_int(dim), _stream(),
        ),
    )
    return out


def min_gru(
    proj: torch.Tensor, z_bias: torch.Tensor, x_bias: torch.Tensor, state: torch.Tensor, batch: Any, out_dtype: torch.dtype,
) -> torch.Tensor:
    """The recurrence of `csrc/min_gru.hip` over the step's tokens.  `proj` [T, 3 * width] (rows may lie apart), or float32
    partial sums [P, T, 3 * width] of it: the gate's, the candidate's and the output gate's projections side by side;
    `z_bias`, `x_bias` float32 [width]; `state` float32 [slots, >= width], read and written at the sequences' slots.
    Returns [T, width] of `out_dtype`: the state times silu(output gate).  A step whose portions all have up to
    `MIN_GRU_WALK` tokens is walked token by token; longer ones run in segments side by side, which differs from the
    walk by float32 rounding."""
    KernelError, _check, _code, _i32, _need_gpu, _ptr, _stream = _base()
    _need_gpu(proj, z_bias, x_bias, state)
    width = z_bias.numel()
    n_partials, partial_stride = 1, 0
    if proj.dim() == 3:
        if proj.dtype != torch.float32 or not proj.is_contiguous():
            raise KernelError("partial sums must be a contiguous float32 [P, T, N] tensor")
        n_partials, n_tokens, ld = proj.shape
        partial_stride = n_tokens * ld
    elif proj.dim() == 2 and proj.stride(1) == 1:
        n_tokens, ld = proj.shape[0], (proj.stride(0) if proj.shape[0] > 1 else proj.shape[1])
    else:
        raise KernelError("the projection must be [T, N] with contiguous rows or partial sums [P, T, N]")
    if proj.shape[-1] < 3 * width or n_tokens != batch.n_tokens:
        raise KernelError(f"the projection {tuple(proj.shape)} must hold {batch.n_tokens} rows of {3 * width}")
    for name, t in (("gate's", z_bias), ("candidate's", x_bias)):
        if t.dtype != torch.float32 or t.shape != (width,) or not t.is_contiguous():
            raise KernelError(f"the {name} bias must be a contiguous float32 [{width}] tensor")
    if state.dtype != torch.float32 or state.dim() != 2 or state.shape[1] < width or not state.is_contiguous():
        raise KernelError(f"the state must be a contiguous float32 [slots, >= {width}] tensor")
    out = torch.empty((n_tokens, width), dtype=out_dtype, device=proj.device)
    segments = step_segments(batch, proj.device, MIN_GRU_WALK, MIN_GRU_SEGMENT, MIN_GRU_SEGMENTS)
    seg_sum = seg_keep = None
    if segments is not None and segments.shape[0] > 65535:
        segments = None  # (more segments than one launch counts: the portions are walked whole)
    if segments is not None:
        seg_sum, seg_keep = (torch.empty((segments.shape[0], width), dtype=torch.float32, device=proj.device) for _ in range(2))
    lib = _build.load("min_gru")
    _check(
        lib,
        lib.cwm_min_gru(
            _ptr(proj), ctypes.c_int(_code(proj.dtype)), ctypes.c_long(ld), ctypes.c_int(n_partials), ctypes.c_long(partial_stride),
            _ptr(z_bias), _ptr(x_bias), _ptr(out), ctypes.c_int(_code(out_dtype)), _ptr(state), ctypes.c_long(state.shape[1]),
            _ptr(batch.state_slots), _ptr(batch.cu_q), ctypes.c_int(state.shape[0]), ctypes.c_int(n_tokens), ctypes.c_int(batch.n_seqs),
            ctypes.c_int(width), _ptr(segments), ctypes.c_int(segments.shape[0] if segments is not None else 0), _ptr(seg_sum), _ptr(seg_keep), _stream(),
        ),
    )
    return out
