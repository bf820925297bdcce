"""The Sunusun architecture on the GPU against the plain implementation.

First the kernels that came with it, each alone against the plain implementation's function for that mechanism
(attention with a distance bias and one added to the softmax's denominator, with a loud key far back and at page
borders; the queries' temperature in the kernel that writes the cache; the gated recurrence and the blends of
neighbouring tokens in portions of any size, with states in slots of any order; linear attention with a bonus, walked
and in blocks on the matrix cores; results normalised before they join the residual; the embedding's positions); then
models: every regime of the replay driver in both types with pages and state slots that are used again; single layers
that leave one mechanism nearly alone; far keys and slow states over long sequences; first tokens and long decoding;
decode steps replayed from graphs; greedy generation through the engine, the command line and `bin/trace_run`; and
configurations drawn from seeds."""

import json
import os
import random
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

from helpers import sunusun, traces
from plain import sunusun_plain as sp

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale


def tolerance(dtype, exact=(2e-5, 2e-5), rounded=(2e-2, 2e-2)):
    return dict(zip(("rtol", "atol"), exact if dtype == torch.float32 else rounded))


def step_batch(lens_old, lens_new, slots=None):
    kv_lens = [a + b for a, b in zip(lens_old, lens_new)]
    cu = [0]
    for n in lens_new:
        cu.append(cu[-1] + n)
    return SimpleNamespace(
        q_lens=list(lens_new), kv_lens=kv_lens, n_seqs=len(kv_lens), n_tokens=sum(lens_new), scratch={}, static=None, max_kv_len=max(kv_lens),
        cu_q=torch.tensor(cu, dtype=torch.int32).to(DEV), kv_len=torch.tensor(kv_lens, dtype=torch.int32).to(DEV),
        positions=torch.cat([torch.arange(a, a + b) for a, b in zip(lens_old, lens_new)]).to(torch.int32).to(DEV),
        seq_of_token=torch.cat([torch.full((n,), b) for b, n in enumerate(lens_new)]).to(torch.int32).to(DEV),
        state_slots=torch.tensor(slots if slots is not None else list(range(len(lens_new))), dtype=torch.int32).to(DEV),
    )


def cut(lengths, sizes):
    """Steps that take the sequences side by side in portions of the given sizes (cycled, each sequence from another place)."""
    cursor, steps, k = [0] * len(lengths), [], 0
    while any(c < n for c, n in zip(cursor, lengths)):
        step = []
        for s, n in enumerate(lengths):
            if cursor[s] < n:
                size = min(sizes[(k + s) % len(sizes)], n - cursor[s])
                step.append((s, cursor[s], cursor[s] + size))
                cursor[s] += size
        steps.append(step)
        k += 1
    return steps


def take(step, slots):
    return step_batch([a for _, a, _ in step], [b - a for _, a, b in step], [slots[s] for s, _, _ in step])


def scatter(got, step, rows):
    at = 0
    for s, a, b in step:
        got[s][a:b] = rows[at : at + b - a]
        at += b - a


# ---- attention with a distance bias --------------------------------------------------------------------------------- #
def _attention_case(dtype, n_q, n_kv, hd, page_size, lens_old, lens_new, seed, loud=(), slope=1.0):
    """Keys, values and queries of a mixed batch in a shuffled paged cache (not a number wherever no key lies), and the
    plain implementation's result."""
    g = torch.Generator().manual_seed(seed)
    scale = hd ** -0.5
    pages_per = [(a + b + page_size - 1) // page_size for a, b in zip(lens_old, lens_new)]
    total = sum(pages_per) + 1
    perm = torch.randperm(total, generator=g)
    table = torch.full((len(lens_old), max(pages_per)), -1, dtype=torch.int32)
    cache = torch.full((total, 2, n_kv, page_size * hd), float("nan"), dtype=dtype)
    vb = 8 if page_size % 8 == 0 else page_size
    kc = cache[:, 0].view(total, n_kv, page_size, hd)
    vc = cache[:, 1].view(total, n_kv, page_size // vb, hd, vb)
    r1, r2 = torch.rand(n_q, generator=g) * 2.0 * slope, torch.rand(n_q, generator=g) * 0.5 + 0.01
    used, q_rows, want_rows, group = 0, [], [], n_q // n_kv
    for b, (n0, n1) in enumerate(zip(lens_old, lens_new)):
        n = n0 + n1
        k, v = torch.randn((n, n_kv, hd), generator=g).to(dtype), torch.randn((n, n_kv, hd), generator=g).to(dtype)
        q = torch.randn((n1, n_q, hd), generator=g).to(dtype)
        for lb, key_pos in loud:
            if lb == b:  # a key that answers the last query's first heads loudly (those of key/value head 0)
                k[key_pos, 0] = (q[-1, 0].float() * 6.0).to(dtype)
        table[b, : pages_per[b]] = perm[used : used + pages_per[b]].to(torch.int32)
        used += pages_per[b]
        pos = torch.arange(n)
        pages, slots = table[b, pos // page_size].long(), pos % page_size
        kc[pages, :, slots, :] = k
        vc[pages, :, slots // vb, :, slots % vb] = v
        at = torch.arange(n)
        scores = torch.einsum("thd,khd->htk", q.double(), k.double().repeat_interleave(group, dim=1)) * scale
        scores = scores - sp.distance_bias(at[n0:], at, r1.double(), r2.double())
        weights = sp.softmax_with_one(scores, at[None, :] <= at[n0:, None])
        want_rows.append(torch.einsum("htk,khd->thd", weights, v.double().repeat_interleave(group, dim=1)).reshape(n1, -1))
        q_rows.append(q)
    bias = (r1.to(DEV), r2.to(DEV))
    return torch.cat(q_rows).to(DEV), cache.to(DEV), table.to(DEV), step_batch(lens_old, lens_new), scale, bias, torch.cat(want_rows)


def _check_attention(dtype, case, what):
    from cwm_amd import ops

    q, cache, table, batch, scale, bias, want = case
    sink = torch.zeros(q.shape[1], dtype=torch.float32, device=DEV)
    got = ops.paged_attention(q, cache, table, batch, None, scale, sink=sink, distance_bias=bias).cpu()
    assert torch.isfinite(got).all(), what
    torch.testing.assert_close(got.double(), want, **tolerance(dtype, (1e-4, 2e-5), (3e-2, 3e-2)), msg=lambda m: f"{what}: {m}")
    return got


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_q,n_kv,hd,page_size", [(4, 2, 16, 8), (3, 1, 32, 16), (12, 2, 128, 64), (6, 3, 80, 16), (5, 5, 48, 5), (8, 2, 64, 32), (9, 3, 112, 12)])
def test_scores_that_fall_with_the_distance(dtype, n_q, n_kv, hd, page_size):
    """Portions beside decoded tokens, after contexts that end inside and at the borders of pages and key tiles; then
    portions of some hundred tokens (the kernel that shares keys through LDS), beside a decoded token."""
    case = _attention_case(dtype, n_q, n_kv, hd, page_size, [0, 131, 300, 17, 255], [40, 1, 3, 1, 2], seed=hd)
    _check_attention(dtype, case, f"{n_q} heads on {n_kv} of {hd}, pages of {page_size}")
    case = _attention_case(dtype, n_q, n_kv, hd, page_size, [0, 131, 70], [200, 1, 330], seed=hd + 1)
    _check_attention(dtype, case, f"long portions: {n_q} heads on {n_kv} of {hd}, pages of {page_size}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [1, 7, 180])
def test_a_loud_key_far_back_among_thousands(dtype, portion):
    """Key ranges that are cut and joined: a loud key in the first of them decides the last query, at a page's first and
    last place; the bias is small enough to leave it loud, and large enough to matter."""
    for place in (3, 63, 64, 1500):
        args = dict(n_q=6, n_kv=2, hd=64, page_size=32, lens_old=[2900 - portion, 700], lens_new=[portion, 5])
        case = _attention_case(dtype, **args, seed=8, loud=[(0, place)], slope=0.3)
        quiet = _attention_case(dtype, **args, seed=8, slope=0.3)
        assert (case[-1][portion - 1] - quiet[-1][portion - 1]).abs().max() > 0.1
        _check_attention(dtype, case, f"a loud key at {place}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_missing_page_gives_nan_and_scores_below_zero_leave_next_to_nothing(dtype):
    from cwm_amd import ops

    q, cache, table, batch, scale, bias, want = _attention_case(dtype, 2, 1, 32, 8, [100], [1], seed=2)
    gone = table.clone()
    gone[0, 4] = -1
    sink = torch.zeros(2, dtype=torch.float32, device=DEV)
    assert torch.isnan(ops.paged_attention(q, cache, gone, batch, None, scale, sink=sink, distance_bias=bias)).any()
    steep = (torch.full((2,), 400.0, device=DEV), torch.full((2,), 1e5, device=DEV))  # every other key's score is far below zero
    got = ops.paged_attention(q, cache, table, batch, None, scale, sink=sink, distance_bias=steep).float().cpu()
    kc = cache[:, 0].view(cache.shape[0], 1, 8, 32)
    own_k = kc[int(table[0, 12]), 0, 100 % 8].double().cpu()
    own = torch.exp((q[0].double().cpu() @ own_k) * scale)
    own_v = cache[:, 1].view(cache.shape[0], 1, 1, 32, 8)[int(table[0, 12]), 0, 0, :, 100 % 8].double().cpu()
    torch.testing.assert_close(got.double().reshape(2, 32), (own / (1.0 + own))[:, None] * own_v[None], **tolerance(dtype, (1e-4, 2e-5), (2e-2, 2e-2)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("coef,every", [(0.5, 7), (-0.2, 1), (0.3, 100)])
def test_the_queries_temperature_touches_queries_only(dtype, coef, every):
    from cwm_amd import ops

    n, n_q, n_kv, qk, vd, hd, page = 9, 3, 1, 12, 10, 16, 8
    positions = torch.tensor([0, 5, 6, 7, 98, 99, 100, 4097, 13], dtype=torch.int32)
    proj = rnd((n, (n_q + n_kv) * qk + n_kv * vd), 1).to(dtype)
    wq, wk = rnd((qk,), 2).abs() + 0.5, rnd((qk,), 3).abs() + 0.5
    table = torch.arange(600, dtype=torch.int32)[None].to(DEV)
    results = []
    for temperature in ((coef, every), None):
        cache = torch.zeros((600, 2, n_kv, page * hd), dtype=dtype, device=DEV)
        q = ops.head_norm_rope_write(proj.to(DEV), n_q, n_kv, qk, vd, hd, None, wq.to(DEV), wk.to(DEV), 1e-5, positions.to(DEV), None, dtype, cache, table,
                                     torch.zeros(n, dtype=torch.int32, device=DEV), temperature=temperature)
        results.append((q.cpu(), cache.cpu()))
    assert torch.equal(results[0][1], results[1][1])
    heads = proj[:, : n_q * qk].double().reshape(n, n_q, qk)
    want = sp.unit_rms(heads, 1e-5) * wq.double() * sp.query_temperature(positions, coef, every)[:, None, None]
    torch.testing.assert_close(results[0][0][..., :qk].double(), want, **tolerance(dtype, (1e-5, 1e-5), (1e-2, 1e-2)))
    assert (results[0][0][..., qk:] == 0).all()


# ---- the gated recurrence -------------------------------------------------------------------------------------------- #
def _recurrence(proj, z_bias, x_bias):
    """The plain rows of one sequence and its last state."""
    width = z_bias.numel()
    z = torch.sigmoid(proj[:, :width] + z_bias)
    c = sp.candidate(proj[:, width : 2 * width] + x_bias)
    state, rows = torch.zeros(width, dtype=F64), []
    for t in range(proj.shape[0]):
        state = (1.0 - z[t]) * state + z[t] * c[t]
        rows.append(state)
    return torch.stack(rows) * sp.silu(proj[:, 2 * width : 3 * width]), state


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [1, 37, 64, 300, 513])
def test_gated_recurrence_in_any_portions(dtype, width):
    """Whole sequences (in segments side by side), portions down to one token, and single tokens; gates nearly shut keep
    the first tokens for hundreds of steps; partial sums of a product are added up."""
    from cwm_amd import ops

    lengths, slots = [700, 5, 64], [2, 0, 3]
    zb, xb = torch.linspace(-9.0, 1.0, width), rnd((width,), 7, 0.5)
    proj = [rnd((n, 3 * width + 2), 3 + i).to(dtype) for i, n in enumerate(lengths)]  # two more columns ride along
    want = [_recurrence(p.double(), zb.double(), xb.double()) for p in proj]
    cuts = {
        "whole": [[(s, 0, n) for s, n in enumerate(lengths)]], "portions": cut(lengths, [64, 2, 33, 1, 130, 32, 31]),
        "two large": [[(0, 0, 301), (1, 0, 5)], [(0, 301, 700), (2, 0, 64)]],
    }
    for what, steps in cuts.items():
        for partial in (False, True):
            state = torch.zeros((4, width + 3), dtype=torch.float32, device=DEV)
            got = [torch.zeros((n, width)) for n in lengths]
            for step in steps:
                p = torch.cat([proj[s][a:b] for s, a, b in step]).to(DEV)
                if partial:
                    share = torch.rand((1, p.shape[1]), generator=torch.Generator().manual_seed(1)).to(DEV)
                    p = torch.stack([p.float() * share, p.float() - p.float() * share])
                scatter(got, step, ops.min_gru(p, zb.to(DEV), xb.to(DEV), state, take(step, slots), dtype).cpu().float())
            for s in range(len(lengths)):
                torch.testing.assert_close(got[s].double(), want[s][0], **tolerance(dtype, (2e-5, 5e-6), (1e-2, 1e-3)), msg=lambda m: f"{what}: {m}")
                torch.testing.assert_close(state[slots[s], :width].cpu().double(), want[s][1], rtol=2e-5, atol=5e-6)
            assert torch.count_nonzero(state[1]) == 0, "a slot that no sequence of the steps names was written"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,offset", [(40, 0), (192, 12), (7, 3), (1100, 4)])
def test_blends_of_neighbouring_tokens_carry_the_last_one(dtype, dim, offset):
    from cwm_amd import ops

    lengths, slots = [23, 5, 40], [3, 1, 0]
    x = [rnd((n, dim), 3 + i).to(dtype) for i, n in enumerate(lengths)]
    mu = rnd((5, dim), 11)
    weights = {f"mu.{s}": m.double() for s, m in zip("rkvgw", mu)}
    want = [torch.stack([sp.token_mixes(weights, "", xs.double())[s] for s in "rkvgw"], dim=1) for xs in x]  # [n, 5, dim]
    state = torch.zeros((4, offset + dim + 1), dtype=torch.float32, device=DEV)
    got = [torch.zeros((n, 5, dim)) for n in lengths]
    for step in cut(lengths, [1, 2, 7, 1, 1, 3, 16]):
        out = ops.token_mixes(torch.cat([x[s][a:b] for s, a, b in step]).to(DEV), mu.to(DEV), state, offset, take(step, slots))
        scatter(got, step, out.cpu().float().transpose(0, 1))
    for s, n in enumerate(lengths):
        torch.testing.assert_close(got[s].double(), want[s], **tolerance(dtype, (1e-5, 1e-5), (1e-2, 1e-2)))
        assert torch.equal(state[slots[s], offset : offset + dim].cpu(), x[s][-1].float())
    assert torch.count_nonzero(state[2]) == 0 and torch.count_nonzero(state[:, :offset]) == 0


# ---- linear attention with a bonus ----------------------------------------------------------------------------------- #
class LinearCase:
    """Inputs of one such linear attention for sequences of given lengths, the kernel's arguments for any cut of the
    sequences into steps, and the plain implementation's results."""

    def __init__(self, heads, dim, lengths, dtype, seed, shift=0.0):
        self.heads, self.dim, self.lengths, self.dtype, self.eps, self.inner = heads, dim, lengths, dtype, 1e-5, heads * dim
        self.parts = [[rnd((n, self.inner), seed + 10 * i + j).to(dtype) for j in range(4)] for i, n in enumerate(lengths)]
        self.z = [rnd((n, self.inner), seed + 50 + i, 1.5) + shift for i, n in enumerate(lengths)]
        self.bonus, self.weight = rnd((self.inner,), seed + 98), rnd((self.inner,), seed + 99).abs() + 0.5

    def reference(self):
        out = []
        for parts, z in zip(self.parts, self.z):
            n = z.shape[0]
            r, k, v, g = (t.double().reshape(n, self.heads, self.dim) for t in parts)
            o = sp.wkv_scan(r, k, v, torch.exp(-torch.exp(z.double())).reshape(n, self.heads, self.dim), self.bonus.double().reshape(self.heads, self.dim))
            out.append(sp.unit_rms(o, self.eps).reshape(n, -1) * self.weight.double() * sp.silu(g).reshape(n, -1))
        return out

    def run(self, steps, slots, n_slots=4):
        from cwm_amd import ops

        state = torch.zeros((n_slots, ops.gla_state_elems(self.heads, self.dim, self.dim) + 4), dtype=torch.float32, device=DEV)
        got = [torch.zeros((n, self.inner)) for n in self.lengths]
        for step in steps:
            parts = [torch.cat([self.parts[s][j][a:b] for s, a, b in step]).to(DEV) for j in range(4)]
            z = torch.cat([self.z[s][a:b] for s, a, b in step]).to(DEV)
            y = ops.wkv(*parts, z, self.bonus.to(DEV), self.weight.to(DEV), state, take(step, slots), self.heads, self.dim, self.dim, self.eps)
            scatter(got, step, y.cpu().float())
        return got, state


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim", [(3, 10), (2, 64), (1, 96), (2, 130), (4, 33), (1, 1), (1, 128), (5, 20)])
def test_linear_attention_with_a_bonus_in_any_portions(dtype, heads, dim):
    """Portions of up to sixteen tokens are walked, with the same bits however a sequence is cut; longer ones in bfloat16
    go in blocks of tokens and segments, with the walk's rows and state but for rounding."""
    lengths, slots = [300, 5, 70], [2, 0, 3]
    case = LinearCase(heads, dim, lengths, dtype, seed=heads * 100 + dim)
    want = case.reference()
    t = tolerance(dtype, (2e-4, 2e-5), (2e-2, 2e-2))
    walked, walked_state = case.run(cut(lengths, [16, 7, 2, 5, 1, 3]), slots)
    again, again_state = case.run(cut(lengths, [3, 11, 16, 1]), slots)
    whole, state = case.run([[(s, 0, n) for s, n in enumerate(lengths)]], slots)
    parts, parts_state = case.run(cut(lengths, [33, 2, 17, 70, 1, 131]), slots)
    assert torch.equal(walked_state, again_state), "a cut of the sequence changed the state's bits"
    for s in range(len(lengths)):
        assert torch.equal(walked[s], again[s]), "a cut of the sequence changed the bits"
        for got in (walked, whole, parts):
            torch.testing.assert_close(got[s].double(), want[s], **t)
    for other in (state, parts_state):
        torch.testing.assert_close(other, walked_state, rtol=2e-4, atol=2e-5)
    assert torch.count_nonzero(state[1]) == 0, "a slot that no sequence of the steps names was written"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shift", [-7.0, 3.0, 9.0])
def test_linear_attention_with_slow_with_fast_and_with_total_decays(dtype, shift):
    """Decays near one keep a loud first token over hundreds of tokens; decays that underflow to zero forget everything
    but the current token, and no quotient of them turns up anywhere."""
    case = LinearCase(2, 24, [400], dtype, seed=7, shift=shift)
    case.parts[0][1][0] *= 8.0  # the first token's keys
    want = case.reference()
    for steps in ([[(0, 0, 400)]], cut([400], [130, 2, 1, 67])):
        got, state = case.run(steps, [0])
        torch.testing.assert_close(got[0].double(), want[0], **tolerance(dtype, (5e-4, 5e-5), (2e-2, 2e-2)))
        assert torch.isfinite(state).all()


@pytest.mark.parametrize("heads,dim,rank,width,batch", [(2, 16, 8, 64, 3), (4, 64, 64, 256, 8), (3, 48, 5, 200, 16), (1, 128, 32, 128, 1), (2, 176, 40, 512, 5), (5, 80, 100, 2048, 8)])
def test_a_decode_step_in_two_kernels(heads, dim, rank, width, batch):
    """The product of five inputs with one joined matrix against five products, with and without the matrix's streaming
    copy; then the kernel from its sums to the gated result against the plain recurrence, over several steps, with
    states in slots of any order."""
    from cwm_amd import ops

    inner, steps, slots = heads * dim, 4, list(range(batch))[::-1]
    w = rnd((4 * inner + rank, width), 1, width ** -0.5).bfloat16()
    w2, w0 = rnd((inner, rank), 2, rank ** -0.5).bfloat16(), rnd((inner,), 3, 2.0) - 1.0
    bonus, weight = rnd((inner,), 4), rnd((inner,), 5).abs() + 0.5
    state = torch.zeros((batch + 1, ops.gla_state_elems(heads, dim, dim) + width), dtype=torch.float32, device=DEV)
    b = step_batch([7] * batch, [1] * batch, slots)
    rows, got = [], []
    for i in range(steps):
        x = rnd((5, batch, width), 10 + i).bfloat16()
        assert ops.linear_inputs_takes(x.to(DEV), w.to(DEV), inner)
        sums = ops.linear_inputs(x.to(DEV), w.to(DEV), inner)
        ends = [0, inner, 2 * inner, 3 * inner, 4 * inner, 4 * inner + rank]
        want = torch.cat([x[j].double() @ w[ends[j] : ends[j + 1]].double().T for j in range(5)], dim=1)
        torch.testing.assert_close(sums.sum(0).cpu().double(), want, rtol=1e-4, atol=1e-4)
        streamed = ops.linear_inputs(x.to(DEV), w.to(DEV), inner, streamed=ops.stream_layout(w.to(DEV)))
        torch.testing.assert_close(streamed, sums, rtol=1e-5, atol=1e-5)
        got.append(ops.wkv_token(sums, w2.to(DEV), w0.to(DEV), bonus.to(DEV), weight.to(DEV), state, b, heads, dim, 1e-5, torch.bfloat16).cpu())
        rows.append(want)
    rows = torch.stack(rows)  # [steps, batch, 4 inner + rank]
    for s in range(batch):
        r, k, v, g = (rows[:, s, j * inner : (j + 1) * inner].reshape(steps, heads, dim) for j in range(4))
        decay = torch.exp(-torch.exp(torch.tanh(rows[:, s, 4 * inner :]) @ w2.double().T + w0.double())).reshape(steps, heads, dim)
        o = sp.wkv_scan(r, k, v, decay, bonus.double().reshape(heads, dim))
        want = sp.unit_rms(o, 1e-5).reshape(steps, -1) * weight.double() * sp.silu(g).reshape(steps, -1)
        torch.testing.assert_close(torch.stack([y[s] for y in got]).double(), want, rtol=1e-2, atol=2e-3)
    assert torch.count_nonzero(state[batch]) == 0, "a slot that no sequence of the steps names was written"


# ---- results that are normalised first, positions, activations -------------------------------------------------------- #
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,addends", [(40, 2), (192, 1), (1024, 2), (2048, 2), (4096, 2), (7, 2), (100, 3), (9000, 2)])
def test_results_are_normalised_before_they_join_the_residual(dtype, dim, addends):
    from cwm_amd import ops

    n, eps_in, eps = 5, 1e-5, 1e-6
    h = rnd((n, dim), 1, 2.0)
    ys = [rnd((n, dim), 10).to(dtype), rnd((6, n, dim), 11), rnd((n, dim + 4), 12).to(dtype)[:, :dim]][:addends]
    ws = [rnd((dim,), 20 + i) for i in range(addends)]
    cs = [0.5, -0.25, 2.0][:addends]
    weight = rnd((dim,), 30).abs() + 0.5
    want = h.double()
    for y, w, c in zip(ys, ws, cs):
        y = y.double().sum(0) if y.dim() == 3 else y.double()
        want = want + c * sp.unit_rms(y, eps_in) * w.double()
    delta = ops.NormedSum([(y.to(DEV), w.to(DEV), c) for y, w, c in zip(ys, ws, cs)], eps_in)
    got = h.clone().to(DEV)
    x = ops.add_normed_rmsnorm(got, delta, weight.to(DEV), eps, dtype).cpu()
    torch.testing.assert_close(got.cpu().double(), want, rtol=2e-5, atol=2e-5)
    torch.testing.assert_close(x.double(), sp.unit_rms(want, eps) * weight.double(), **tolerance(dtype, (2e-5, 2e-5), (1e-2, 1e-2)))
    rows = torch.tensor([4, 0, 2], dtype=torch.int32, device=DEV)
    kept = h.clone().to(DEV)
    some = ops.add_normed_rmsnorm(kept, delta, weight.to(DEV), eps, dtype, rows).cpu()
    assert torch.equal(kept.cpu(), h)
    torch.testing.assert_close(some, x[rows.long().cpu()], rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [40, 7, 1026])
def test_embedding_with_sinusoidal_positions(dtype, dim):
    from cwm_amd.parts.base import Runtime
    from cwm_amd.parts.embedding import SinusoidalTokenEmbedding

    table = rnd((30, dim), 1).to(dtype)
    positions = torch.tensor([0, 1, 2, 63, 64, 1000, 131071, 1000003], dtype=torch.int32)
    tokens = torch.tensor([3, 3, 0, 29, 7, 8, 9, 10], dtype=torch.int32)
    part = SinusoidalTokenEmbedding(30, dim, 10000.0, scale=0.5, tensor="")
    part.bind({"": table.to(DEV)}, Runtime(device=torch.device(DEV), act_dtype=dtype))
    got = part.forward(SimpleNamespace(tokens=tokens.to(DEV), positions=positions.to(DEV))).cpu()
    torch.testing.assert_close(got.double(), 0.5 * table[tokens.long()].double() + sp.sinusoid(positions, dim), rtol=1e-6, atol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
def test_erf_gelu_and_tanh_on_rows(dtype):
    from cwm_amd import ops

    x = torch.cat([torch.linspace(-7.0, 7.0, 300), rnd((84,), 1)]).reshape(4, 96)
    for kind, f in (("gelu_erf", sp.gelu_erf), ("tanh", torch.tanh)):
        torch.testing.assert_close(ops.act_rows(x.to(dtype).to(DEV), kind, dtype).cpu().double(), f(x.to(dtype).double()), **tolerance(dtype, (2e-6, 1e-6), (1e-2, 1e-3)))
        parts = torch.stack([x * 0.25, x * 0.75]).to(DEV)
        torch.testing.assert_close(ops.act_rows(parts, kind, torch.float32).cpu().double(), f(x.double()), rtol=2e-6, atol=1e-6)


# ---- models through the replay driver ------------------------------------------------------------------------------------ #
LENGTHS = {"tiny_j": [1, 6, 21, 40, 90], "tiny_k": [9, 33, 2, 70, 26], "tiny_l": [120, 12, 45, 64]}
PAGE_SIZES = {"whole": 16, "tail": 32, "portions": 8, "mixed": 12}


def requests_for(name, lengths=None):
    vocab = sunusun.get(name)["vocab"]
    return {f"r{i}": traces.random_tokens(17 * i + len(name), n, vocab) for i, n in enumerate(lengths or LENGTHS[name])}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("sunusun")
    return {name: sunusun.make_folder(root, name, seed=5) for name in sunusun.ALL}


@pytest.fixture(scope="module")
def plain_cache():
    return {}


def plain_for(folders, cache, name, dtype):
    if (name, dtype) not in cache:
        cache[name, dtype] = sunusun.expected(folders[name], requests_for(name), dtype, conditioning=True)
    return cache[name, dtype]


def run(folder, dtype, steps, requests, vocab, **options):
    from cwm_amd.replay import Replayer

    rep = Replayer(folder, dtype, traces.max_live_tokens(steps), poison_freed_pages=True, **options)
    page_use = traces.PageUse(rep.manager)
    outputs = traces.run_in_process(rep, steps, page_use)
    assert rep.manager.live_requests() == []
    return traces.gather(steps, outputs, {k: len(v) for k, v in requests.items()}, vocab), rep, page_use


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(sunusun.ALL))
@pytest.mark.parametrize("regime", ["whole", "tail", "portions", "mixed"])
def test_replay_regimes(folders, plain_cache, name, dtype, regime):
    requests = requests_for(name)
    vocab = sunusun.get(name)["vocab"]
    steps = {"whole": traces.whole, "tail": traces.tail_one_by_one, "portions": traces.portions,
             "mixed": lambda r: traces.mixed(r, max_live=3)}[regime](requests)
    got, rep, page_use = run(folders[name], dtype, steps, requests, vocab, page_size=PAGE_SIZES[regime], max_requests=3 if regime == "mixed" else 16)
    sunusun.check_together(got, plain_for(folders, plain_cache, name, dtype), dtype, f"{name} {dtype} {regime}")
    if regime == "mixed":
        for g in rep.manager.groups:
            assert page_use.pages_shared_between_requests(g.index) > 0, f"group {g.index}: no page served two requests"


P, W = sunusun.parallel, sunusun.wkv
SINGLE_LAYERS = {
    "parallel": dict(layers=[P(4, 2, 12, 10, 0.3, 30, temp=(0.5, 5))]),
    "parallel_without_temperature": dict(layers=[P(3, 3, 8, 16, 0.4, 9, mlp=24)]),
    "parallel_with_narrow_heads_and_a_wide_state": dict(layers=[P(2, 1, 6, 6, 1.0, 130, temp=(0.3, 2))], eps=1e-3),
    "wkv": dict(layers=[W(3, 10)]),
    "wkv_with_one_wide_head": dict(layers=[W(1, 100, mlp=16)], logit_scale=0.3),
    "one_layer_run_three_times": dict(layers=[W(2, 18, mlp=12), W(0, 0, weights_of=0), W(0, 0, weights_of=1)]),
    "parallel_run_twice": dict(layers=[P(2, 2, 10, 14, 0.3, 25, temp=(0.2, 9), mlp=20), P(0, 0, 0, 0, 0, 0, weights_of=0)]),
    "no_feed_forward_anywhere": dict(layers=[P(1, 1, 8, 8, 0.3, 12, temp=(0.2, 9)), W(2, 8), P(1, 1, 8, 8, 0.3, 12)], width=36),
    "feed_forward_carries_the_layer": dict(layers=[W(1, 4, mlp=100)], width=24),
    "an_odd_width": dict(layers=[P(2, 1, 7, 5, 0.3, 11, temp=(0.2, 3), mlp=13), W(2, 5, mlp=9)], width=27),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", list(SINGLE_LAYERS))
def test_single_layers(tmp_path, which, dtype):
    """One mechanism at a time between embedding and head: whole prompts against the same tokens in portions and one by
    one, and all against the plain implementation."""
    config = sunusun.model_of(**SINGLE_LAYERS[which])
    folder = sunusun.make_folder(tmp_path, which[:40], seed=2, config=config)
    requests = {f"r{i}": traces.random_tokens(i + 5, n, config["vocab"]) for i, n in enumerate([37, 5, 64])}
    want = sunusun.expected(folder, requests, dtype)
    for make in (traces.whole, traces.portions, lambda r: traces.tail_one_by_one(r, tail=20)):
        steps = make(requests)
        got, _, _ = run(folder, dtype, steps, requests, config["vocab"], page_size=8)
        sunusun.check_together(got, want, dtype, f"{which} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_and_slow_states_over_long_sequences(folders, dtype):
    """tiny_k's softmax is sharp and its states forget slowly: a token's result hangs on single keys, near and far, and on
    what the states took in at the sequence's start.  A prompt of 500 tokens whole, in portions that end at, before and
    after page borders (down to one and two tokens), and with its last 120 tokens one by one."""
    name = "tiny_k"
    vocab = sunusun.get(name)["vocab"]
    requests = {"long": traces.random_tokens(99, 500, vocab)}
    want = sunusun.expected(folders[name], requests, dtype, conditioning=True)
    portions = lambda r: traces.portions(r, sizes=[64, 63, 65, 2, 126, 1, 31, 33, 128, 17, 11, 5, 16])  # noqa: E731
    for make in (traces.whole, portions, lambda r: traces.tail_one_by_one(r, tail=120)):
        steps = make(requests)
        got, _, _ = run(folders[name], dtype, steps, requests, vocab, page_size=32)
        sunusun.check(got["long"], want["long"], dtype, f"{name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_wider_layers_and_many_rows(tmp_path, dtype):
    """Prompts of 500 and 300 tokens: the kernels' shapes for many rows, whole, in large portions beside each other, and
    with a tail of single tokens."""
    config = sunusun.MEDIUM
    folder = sunusun.make_folder(tmp_path, "medium", seed=9, config=config)
    vocab = config["vocab"]
    requests = {"a": traces.random_tokens(31, 500, vocab), "b": traces.random_tokens(32, 300, vocab)}
    want = sunusun.expected(folder, requests, dtype)
    side_by_side = [
        {"step": 0, "entries": [{"id": "a", "tokens": requests["a"][:290], "want": list(range(290))}, {"id": "b", "tokens": requests["b"][:270], "want": list(range(270))}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": requests["a"][290:], "want": list(range(210))}, {"id": "b", "tokens": requests["b"][270:], "want": list(range(30))}], "end": ["a", "b"]},
    ]
    for steps in (traces.whole(requests), side_by_side, traces.tail_one_by_one(requests, tail=20)):
        got, _, _ = run(folder, dtype, steps, requests, vocab, page_size=32)
        sunusun.check_together(got, want, dtype, f"medium {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_and_long_decoding(folders, dtype):
    """Every token a step of its own from an empty cache and zero states, for 250 steps."""
    name = "tiny_j"
    vocab = sunusun.get(name)["vocab"]
    requests = {"a": traces.random_tokens(4, 250, vocab)}
    steps = traces.tail_one_by_one(requests, tail=249)
    got, _, _ = run(folders[name], dtype, steps, requests, vocab, page_size=16)
    sunusun.check(got["a"], sunusun.expected(folders[name], requests, dtype, conditioning=True)["a"], dtype, f"{name} {dtype} one by one")


def test_pages_and_state_slots_that_are_used_again_start_afresh(folders):
    """One slot and a pool of the longer request's size only: the second request finds the first one's states and cache
    rows (NaN in the pages in between) and must not read them."""
    name = "tiny_l"
    vocab = sunusun.get(name)["vocab"]
    a, b = traces.random_tokens(1, 60, vocab), traces.random_tokens(2, 25, vocab)
    both = [
        {"step": 0, "entries": [{"id": "a", "tokens": a, "want": [59]}], "end": ["a"]},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:10], "want": list(range(10))}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[10:], "want": list(range(15))}], "end": ["b"]},
    ]
    got, rep, _ = run(folders[name], "float32", both, {"a": a, "b": b}, vocab, page_size=8, max_requests=1)
    alone, _, _ = run(folders[name], "float32", both[1:], {"b": b}, vocab, page_size=8, max_requests=1)
    assert np.array_equal(got["b"], alone["b"])
    sunusun.check(got["b"], sunusun.expected(folders[name], {"b": b}, "float32")["b"], "float32", "second user of the slot")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_do_not_depend_on_the_rest_of_the_batch(folders, dtype):
    """A request's decoded tokens alone, beside two other requests' short portions, and beside a long one."""
    name = "tiny_j"
    vocab = sunusun.get(name)["vocab"]
    r = requests_for(name, [40, 64, 90, 400])
    head = {"step": 0, "entries": [{"id": "r0", "tokens": r["r0"][:30], "want": [29]}], "end": []}
    alone = [head] + [{"step": 1 + i, "entries": [{"id": "r0", "tokens": [r["r0"][30 + i]], "want": [0]}], "end": ["r0"] if i == 9 else []} for i in range(10)]
    beside, long = [head], [head]
    for i in range(10):
        own = {"id": "r0", "tokens": [r["r0"][30 + i]], "want": [0]}
        beside.append({"step": 1 + i, "entries": [{"id": "r1", "tokens": r["r1"][6 * i : 6 * i + 6], "want": [5]}, own, {"id": "r2", "tokens": r["r2"][8 * i : 8 * i + 8], "want": []}],
                       "end": ["r0", "r1", "r2"] if i == 9 else []})
        long.append({"step": 1 + i, "entries": [own, {"id": "r3", "tokens": r["r3"][40 * i : 40 * i + 40], "want": []}], "end": ["r0", "r3"] if i == 9 else []})
    want = sunusun.expected(folders[name], {"r0": r["r0"]}, dtype, conditioning=True)["r0"]
    rows = {}
    for what, steps in (("alone", alone), ("beside", beside), ("long", long)):
        got, _, _ = run(folders[name], dtype, steps, r, vocab, page_size=8)
        rows[what] = got["r0"][29:]
        size = float(np.abs(want.exact).max())
        np.testing.assert_allclose(rows[what], want.exact[29:], atol=(1e-4 if dtype == "float32" else 0.08) * size, rtol=0)
    for what in ("beside", "long"):
        np.testing.assert_allclose(rows[what], rows["alone"], atol=(2e-5 if dtype == "float32" else 0.05) * float(np.abs(want.exact).max()), rtol=0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["tiny_j", "tiny_k"])
def test_decode_steps_replayed_from_graphs_give_the_same_bits(folders, name, dtype):
    vocab = sunusun.get(name)["vocab"]
    requests = requests_for(name, [30, 44, 37])
    heads = {"step": 0, "entries": [{"id": r, "tokens": t[:20], "want": [19]} for r, t in requests.items()], "end": []}
    steps = [heads] + [
        {"step": 1 + i, "entries": [{"id": r, "tokens": [t[20 + i]], "want": [0]} for r, t in requests.items()], "end": list(requests) if i == 9 else []}
        for i in range(10)
    ]
    launched, _, _ = run(folders[name], dtype, steps, {k: v[:30] for k, v in requests.items()}, vocab, page_size=16)
    replayed, rep, _ = run(folders[name], dtype, steps, {k: v[:30] for k, v in requests.items()}, vocab, page_size=16, num_graphs=2)
    assert rep.runner.n_replays >= 8, "the decode steps were not replayed"
    for rid in requests:
        assert np.array_equal(launched[rid][19:], replayed[rid][19:]), rid


@pytest.mark.parametrize("name", ["tiny_j", "tiny_l"])
def test_greedy_generation_through_the_engine(folders, name):
    """The engine's own entry point: scheduler, portions of 24 tokens, continuous batching, sampling kernel; then a cache
    that holds barely more than the longest request, so that requests wait for one another's pages and slots."""
    from cwm_amd.engine import Engine, GenArgs

    vocab = sunusun.get(name)["vocab"]
    prompts = [traces.random_tokens(20 + i, n, vocab) for i, n in enumerate([5, 17, 33, 64])]
    engine = Engine.from_folder(folders[name], GenArgs(use_sampling=False, max_batch=4, max_seq=2048, cache_block=16, max_prefill=24), dtype="float32")
    got = engine.generate_tokens(prompts, max_gen=12)
    for p, g in zip(prompts, got):
        assert g == sunusun.plain_greedy(folders[name], p, 12)
    small = Engine.from_folder(folders[name], GenArgs(use_sampling=False, max_batch=4, max_seq=96, cache_block=4, max_prefill=24), dtype="float32")
    assert small.generate_tokens(prompts, max_gen=12) == got


def test_command_line_and_trace_run_as_child_processes(folders, tmp_path):
    name = "tiny_j"
    vocab = sunusun.get(name)["vocab"]
    prompts = [traces.random_tokens(60 + i, n, vocab) for i, n in enumerate([6, 21])]
    path = tmp_path / "prompts.jsonl"
    path.write_text("".join(json.dumps({"id": i, "tokens": p}) + "\n" for i, p in enumerate(prompts)))
    cmd = [sys.executable, "-m", "cwm_amd.generate", f"checkpoint_dir={folders[name]}", f"prompts={path}", "dtype=float32",
           "gen_args.use_sampling=false", "gen_args.max_gen=7", "gen_args.max_seq=512", "gen_args.cache_block=16", "gen_args.max_batch=4"]
    res = subprocess.run(cmd, cwd=ROOT, capture_output=True, text=True, timeout=300)
    assert res.returncode == 0, res.stderr
    got = {rec["id"]: rec["tokens"] for rec in map(json.loads, res.stdout.strip().splitlines())}
    for i, p in enumerate(prompts):
        assert got[i] == sunusun.plain_greedy(folders[name], p, 7)

    requests = requests_for(name, [40, 75, 33, 5, 60])
    steps = traces.mixed(requests)
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / f"out_{dtype}"
        cmd = [os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name], "--dtype", dtype, "--out", str(out),
               "--max-tokens", str(traces.max_live_tokens(steps))]
        res = subprocess.run(cmd, input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
        assert res.returncode == 0, res.stderr
        assert [line for line in res.stdout.splitlines() if line.startswith("done")] == [f"done {s['step']}" for s in steps]
        outputs = {s["step"]: np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(-1, vocab) for s in steps if any(e["want"] for e in s["entries"])}
        got = traces.gather(steps, outputs, {k: len(v) for k, v in requests.items()}, vocab)
        sunusun.check_together(got, sunusun.expected(folders[name], requests, dtype), dtype, f"trace_run {dtype}")


def random_config(seed):
    rng = random.Random(1000 + seed)
    width = rng.choice([24, 40, 64, 72, 100, 160])
    layers = []
    for i in range(rng.randint(1, 5)):
        if layers and rng.random() < 0.25:
            j = rng.randrange(len(layers))
            layers.append(dict(P(0, 0, 0, 0, 0, 0, weights_of=j) if layers[j]["type"] == "parallel" else W(0, 0, weights_of=j)))
            continue
        mlp = rng.choice([None, 12, 40, 130])
        if rng.random() < 0.5:
            layers.append(W(rng.randint(1, 5), rng.choice([3, 8, 16, 31, 48, 64, 90]), mlp=mlp))
        else:
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([6, 8, 16, 24, 40, 64, 100])
            temp = rng.choice([None, (0.3, rng.choice([1, 5, 16, 33, 64])), (-0.1, 20)])
            layers.append(P(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([5, 8, 16, 32, 80, 128]), rng.choice([0.1, 0.3]) * (64 / dim) ** 0.5, rng.choice([1, 16, 50, 131]), temp=temp, mlp=mlp))
    return sunusun.model_of(layers, width=width, vocab=rng.randint(50, 700), eps=rng.choice([1e-5, 1e-6]), logit_scale=rng.choice([0.3, 1.0, 2.5]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(tmp_path, seed, dtype):
    """Other models of the design: whole prompts, and a mixed schedule with pages of another size, against the plain
    implementation."""
    config = random_config(seed)
    folder = sunusun.make_folder(tmp_path, f"random{seed}", seed=seed, config=config)
    vocab = config["vocab"]
    requests = {f"r{i}": traces.random_tokens(7 * seed + i, n, vocab) for i, n in enumerate([3, 130, 45, 88])}
    want = sunusun.expected(folder, requests, dtype, conditioning=True)
    for steps, page in ((traces.whole(requests), 16), (traces.mixed(requests, max_live=3), 32 if seed % 2 else 8)):
        got, _, _ = run(folder, dtype, steps, requests, vocab, page_size=page, max_requests=4)
        sunusun.check_together(got, want, dtype, f"random configuration {seed} {dtype}: {json.dumps(config)}")
