"""The Sorovik architecture on the GPU against the plain implementation.

First the kernels that came with it, each alone against the plain implementation's function for that mechanism
(attention over a window and kept first tokens, in both attention kernels and every shape of theirs, with loud keys at the
edges of both; rows of a cached latent; queries and keys behind a convolution in portions of any size, with states in
slots that are used again; a router with groups; normalised sums of routed experts); then models: every regime of the replay
driver in both types with pages and state slots that are used again; single layers that leave one mechanism nearly
alone; sharp attention over long sequences; first tokens and long decoding; decode steps replayed from graphs; greedy
generation through the engine, the command line and `bin/trace_run`; and configurations drawn from seeds."""

import json
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

from helpers import cache_layout, sorovik, traces
from plain import sorovik_plain as sp

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rnd(shape, seed, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(shape, generator=g) * scale


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
    cursor = [0] * len(lengths)
    steps, k = [], 0
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


# ---- attention over a window and kept first tokens ------------------------------------------------------------------ #
class KeptCase:
    """Queries, keys and values of a mixed batch in a shuffled paged cache whose unread pages and slots hold NaN, and the
    plain implementation's result.  `loud`: (sequence, key) pairs, keys that answer their sequence's last query loudly."""

    def __init__(self, dtype, n_q, n_kv, hd, page_size, lens_old, lens_new, window, keep, seed, loud=(), scaled=True):
        g = torch.Generator().manual_seed(seed)
        self.dtype, self.window, self.keep, self.scale = dtype, window, keep, hd ** -0.5
        pages_per = [(a + b + page_size - 1) // page_size for a, b in zip(lens_old, lens_new)]
        total = sum(pages_per) + 1
        perm = torch.randperm(total, generator=g)
        table = torch.full((len(lens_old), max(pages_per)), -1, dtype=torch.int32)
        cache = torch.full((total, 2, n_kv, page_size * hd), float("nan"), dtype=dtype)
        sink = torch.zeros(n_q)
        factor = torch.rand((sum(lens_new), n_q), generator=g) + 0.25
        used, row, q_rows, want = 0, 0, [], []
        for b, (n0, n1) in enumerate(zip(lens_old, lens_new)):
            n = n0 + n1
            k, v = torch.randn((n, n_kv, hd), generator=g).to(dtype), torch.randn((n, n_kv, hd), generator=g).to(dtype)
            q = torch.randn((n1, n_q, hd), generator=g).to(dtype)
            for lb, key in loud:
                if lb == b:
                    k[key, 0] = (q[-1, 0].float() * 6.0).to(dtype)
            visible = sp.visible_keys(n, window, keep)[n0:]
            for key in torch.nonzero(visible.any(0))[:, 0].tolist():  # keys that no query of the step reads stay NaN, their pages missing
                lp = key // page_size
                if table[b, lp] < 0:
                    table[b, lp] = perm[used]
                    used += 1
                cache_layout.write_kv(cache, int(table[b, lp]), key % page_size, k[key], v[key], hd)
            scores = torch.einsum("thd,khd->htk", q.double(), k.double().repeat_interleave(n_q // n_kv, dim=1)) * self.scale
            w = sp.sink_softmax(scores, visible, sink.double())
            out = torch.einsum("htk,khd->thd", w, v.double().repeat_interleave(n_q // n_kv, dim=1))
            want.append((out * factor[row : row + n1, :, None].double() if scaled else out).reshape(n1, -1))
            q_rows.append(q)
            row += n1
        self.q, self.cache, self.table = torch.cat(q_rows).to(DEV), cache.to(DEV), table.to(DEV)
        self.sink, self.factor = sink.to(DEV), factor.contiguous().to(DEV) if scaled else None
        self.batch, self.want = step_batch(lens_old, lens_new), torch.cat(want)

    def check(self, what):
        from cwm_amd import ops

        t = dict(rtol=1e-4, atol=2e-5) if self.dtype == torch.float32 else dict(rtol=3e-2, atol=3e-2)
        args = dict(sink=self.sink, keep_first=self.keep, out_scale=self.factor)
        got = ops.paged_attention(self.q, self.cache, self.table, self.batch, self.window, self.scale, **args).cpu()
        torch.testing.assert_close(got.double(), self.want, **t, msg=lambda m: f"{what}: {m}")
        plain = ops.paged_attention_simple(self.q, self.cache, self.table, self.batch.positions, self.batch.seq_of_token, self.window, self.scale,
                                           max_keys=self.batch.max_kv_len, **args).cpu()
        torch.testing.assert_close(plain.double(), self.want, **t, msg=lambda m: f"{what}, the plain kernel: {m}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(1, 1), (7, 3), (40, 33), (100, 5), (128, 64), (33, 100), (300, 31)])
@pytest.mark.parametrize("n_q,n_kv,hd,page_size", [(4, 2, 16, 8), (12, 2, 128, 64), (6, 3, 80, 16), (5, 5, 48, 5), (8, 1, 64, 32), (3, 1, 192, 32)])
def test_kept_first_tokens_beside_a_window(dtype, n_q, n_kv, hd, page_size, window, keep):
    """Decoded tokens, short portions and long ones (whose blocks share keys through LDS) beside each other, after contexts
    that end inside and at the borders of pages, tiles and the kept tokens; pages between kept tokens and windows are gone."""
    case = KeptCase(dtype, n_q, n_kv, hd, page_size, [0, 331, 400, 17, 255, 90], [40, 1, 3, 1, 2, 310], window, keep, seed=hd + window)
    case.check(f"{n_q} heads on {n_kv} of {hd}, pages of {page_size}, window {window}, {keep} kept")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [1, 9, 300])
@pytest.mark.parametrize("window,keep,page_size", [(64, 16, 16), (40, 33, 32), (2, 5, 8), (129, 64, 64)])
def test_a_loud_key_at_the_edges_of_window_and_kept_tokens(dtype, window, keep, page_size, portion):
    """A key that answers the last query loudly: the last kept token and the window's first place carry the result, one
    place after and one place before them change nothing."""
    last = 3 * window + 2 * keep + 5 + 300
    olds, news = [last + 1 - portion, 9], [portion, 4]
    make = lambda *keys: KeptCase(dtype, 4, 2, 64, page_size, olds, news, window, keep, 3, loud=[(0, key) for key in keys])  # noqa: E731
    quiet = make()
    for key, seen in ((keep - 1, True), (keep, False), (last - window + 1, True), (last - window, False), (0, True)):
        case = make(key)
        case.check(f"loud key {key}, window {window}, {keep} kept, portion {portion}")
        moved = float((case.want[portion - 1] - quiet.want[portion - 1]).abs().max())
        assert moved > 0.1 if seen else moved == 0.0


@pytest.mark.parametrize("dtype", DTYPES)
def test_kept_tokens_before_windows_of_thousands(dtype):
    """Windows that are cut into ranges (and joined again): the kept tokens count once, for a decoded token, a short portion
    and a long one."""
    case = KeptCase(dtype, 4, 2, 64, 32, [6000, 5500, 4000], [1, 5, 200], 5000, 70, seed=8, loud=[(0, 69), (1, 3), (2, 0)])
    case.check("windows of 5,000 keys, 70 kept")
    fine = KeptCase(dtype, 8, 1, 128, 64, [9000], [40], 8300, 40, seed=9, loud=[(0, 39)])
    fine.check("a portion whose window is cut at fixed places, 40 kept")


def test_a_factor_on_every_head_without_kept_tokens():
    for dtype in DTYPES:
        KeptCase(dtype, 4, 2, 32, 16, [0, 50, 3000], [150, 1, 1], 2900, 0, seed=4).check(f"{dtype} factor")


def test_a_missing_page_of_a_kept_token_gives_nan():
    from cwm_amd import ops

    for dtype in DTYPES:
        case = KeptCase(dtype, 2, 1, 16, 8, [100], [1], 30, 9, seed=2, scaled=False)
        gone = case.table.clone()
        gone[0, 1] = -1  # keys 8..15: the last kept one
        got = ops.paged_attention(case.q, case.cache, gone, case.batch, 30, case.scale, sink=case.sink, keep_first=9)
        assert torch.isnan(got).any()
        case.check("nothing missing")


# ---- rows of a cached latent ---------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,lead,rest,rank,page_size,parts", [(3, 6, 10, 12, 8, 1), (5, 16, 24, 64, 16, 3), (16, 64, 128, 192, 32, 4), (1, 0, 7, 33, 5, 1), (2, 2, 4, 30, 16, 2)])
def test_rows_of_a_cached_latent(dtype, heads, lead, rest, rank, page_size, parts):
    """A mixed batch: cached rows, rotated and unrotated query parts from a joined product, stored or in partial sums."""
    from cwm_amd import ops

    row = -(-(lead + rank) // 16) * 16
    lens_old, lens_new = [0, 37, 90], [21, 1, 600 if heads == 3 else 5]
    batch = step_batch(lens_old, lens_new)
    n = batch.n_tokens
    width = lead + rank + heads * (lead + rest)
    proj = rnd((parts, n, width), 1)
    proj = proj[0].to(dtype) if parts == 1 else proj
    total = proj.double() if parts == 1 else proj.double().sum(0)
    weight, freq = rnd((rank,), 2).abs() + 0.5, rnd((max(1, lead // 2),), 3).abs()
    pages_per = [(a + b + page_size - 1) // page_size for a, b in zip(lens_old, lens_new)]
    table = torch.full((3, max(pages_per)), -1, dtype=torch.int32)
    for b, count in enumerate(pages_per):
        table[b, :count] = torch.arange(count) + sum(pages_per[:b])
    cache = torch.zeros((sum(pages_per), 2, 1, page_size * row), dtype=dtype, device=DEV)
    dev = proj.to(DEV)
    ask, un = ops.latent_rows(dev[..., lead + rank :], dev[..., : lead + rank], heads, lead, rest, rank, row, weight.to(DEV), 1e-5, batch, freq.to(DEV), dtype, cache, table.to(DEV))
    angle = batch.positions.cpu().double()[:, None] * freq.double()[None, :]

    def turn(x):  # adjacent pairs
        c, s = torch.cos(angle)[:, None, : lead // 2], torch.sin(angle)[:, None, : lead // 2]
        re, im = x[..., 0::2], x[..., 1::2]
        return torch.stack([re * c - im * s, im * c + re * s], dim=-1).flatten(-2)

    q = total[:, lead + rank :].reshape(n, heads, lead + rest)
    t = dict(rtol=1e-4, atol=1e-4) if dtype == torch.float32 else dict(rtol=1e-2, atol=3e-2)
    torch.testing.assert_close(ask[:, :, :lead].cpu().double(), turn(q[:, :, :lead]), **t)
    torch.testing.assert_close(un.cpu().double(), q[:, :, lead:], **t)
    c = sp.unit_rms(total[:, lead : lead + rank], 1e-5) * weight.double()
    want = torch.cat([turn(total[:, None, :lead])[:, 0], c, torch.zeros(n, row - lead - rank, dtype=torch.float64)], dim=1)
    host = cache.cpu()
    for i in range(n):
        b, p = int(batch.seq_of_token[i]), int(batch.positions[i])
        k, v = cache_layout.read_kv(host, int(table[b, p // page_size]), p % page_size, row)
        torch.testing.assert_close(k[0].double(), want[i], **t)
        assert torch.equal(k, v)
    # a layer that reads another's rows: the queries alone, the same bits
    again, _ = ops.latent_rows(dev[..., lead + rank :], None, heads, lead, rest, rank, row, None, 1e-5, batch, freq.to(DEV), dtype)
    assert torch.equal(again[:, :, :lead], ask[:, :, :lead])


# ---- queries and keys behind a convolution -------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_q,n_kv,dim,taps,parts,lengths", [(4, 2, 12, 3, 1, [23, 5, 40]), (3, 1, 7, 4, 2, [23, 5, 40]), (2, 2, 80, 1, 3, [9, 4, 17]), (3, 3, 16, 9, 1, [23, 5, 40]),
                                                             (8, 2, 64, 2, 1, [700, 3, 900]), (6, 3, 10, 4, 1, [1300, 2, 31])])
def test_convolved_queries_and_keys_in_any_portions(dtype, n_q, n_kv, dim, taps, parts, lengths):
    """Portions shorter and longer than the taps, steps of single tokens (which move their state themselves) and steps of
    many tokens, in slots of any order: queries, cached keys and values, gates and states of the plain implementation."""
    from cwm_amd import ops

    page_size, head_dim, eps = 16, -(-dim // 16) * 16, 1e-5
    channels = (n_q + n_kv) * dim
    proj = [rnd((parts, n, channels + n_q), 5 + i) for i, n in enumerate(lengths)]
    if parts == 1:
        proj = [p.to(dtype).float() for p in proj]
    bias, w = rnd((channels,), 11, 0.5), rnd((channels, taps), 12)
    qw, kw = rnd((n_q * dim,), 13).abs() + 0.5, rnd((n_kv * dim,), 14).abs() + 0.5
    freq = torch.zeros(head_dim // 2)
    freq[: dim // 4] = rnd((dim // 4,), 15).abs().clamp(max=1.0) * (1.0 if max(lengths) < 100 else 0.1)  # far angles are coarse in float32
    slots = [3, 1, 0]
    state = torch.zeros((4, max(1, (taps - 1) * channels)), device=DEV)
    pages_per = [-(-n // page_size) for n in lengths]
    tables = [torch.arange(c, dtype=torch.int32) + sum(pages_per[:b]) for b, c in enumerate(pages_per)]
    cache = torch.zeros((sum(pages_per), 2, n_kv, page_size * head_dim), dtype=dtype, device=DEV)
    got_q, got_g = [torch.zeros((n, n_q, head_dim)) for n in lengths], [torch.zeros((n, n_q)) for n in lengths]
    sizes = [1, 2, 7, 1, 1, 3, 16] if max(lengths) < 100 else [450, 1, 900, 3, 1100]
    steps = cut(lengths, sizes)
    if max(lengths) < 100:
        steps = cut([min(n, 3) for n in lengths], [1]) + [[(s, a + min(lengths[s], 3), b + min(lengths[s], 3)) for s, a, b in step] for step in cut([max(0, n - 3) for n in lengths], sizes)]
    for step in steps:
        batch = step_batch([a for _, a, _ in step], [b - a for _, a, b in step], [slots[s] for s, _, _ in step])
        table = torch.full((len(step), max(pages_per)), -1, dtype=torch.int32)
        for i, (s, _, _) in enumerate(step):
            table[i, : pages_per[s]] = tables[s]
        x = torch.cat([proj[s][:, a:b] for s, a, b in step], dim=1).contiguous()
        x = x[0].to(dtype) if parts == 1 else x
        q, gates = ops.conv_qk_rope_write(x.to(DEV), n_q, n_kv, dim, head_dim, bias.to(DEV), w.t().contiguous().to(DEV), qw.to(DEV), kw.to(DEV), eps, batch,
                                          freq.to(DEV), dtype, cache, table.to(DEV), state if taps > 1 else None, gate=True)
        row = 0
        for s, a, b in step:
            got_q[s][a:b], got_g[s][a:b] = q[row : row + b - a].cpu().float(), gates[row : row + b - a].cpu()
            row += b - a
    t = dict(rtol=2e-4, atol=2e-4) if dtype == torch.float32 else dict(rtol=2e-2, atol=3e-2)
    host = cache.cpu()
    for s, n in enumerate(lengths):
        total = proj[s].double().sum(0)
        u = total[:, :channels] + bias.double()
        y = sp.causal_conv(u, w.double())
        angle = torch.arange(n).double()[:, None] * freq.double()[None, :]
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]

        def ready(x, heads, weight):
            x = (sp.unit_rms(x, eps) * weight.double()).reshape(n, heads, dim)
            x = torch.nn.functional.pad(x, (0, head_dim - dim))
            re, im = x[..., 0::2], x[..., 1::2]
            return torch.stack([re * cos - im * sin, im * cos + re * sin], dim=-1).flatten(-2)

        torch.testing.assert_close(got_q[s].double(), ready(y[:, : n_q * dim], n_q, qw), **t)
        torch.testing.assert_close(got_g[s].double(), torch.sigmoid(total[:, channels:]), rtol=1e-4, atol=1e-5)
        keys, values = ready(y[:, n_q * dim :], n_kv, kw), torch.nn.functional.pad(y[:, n_q * dim :].reshape(n, n_kv, dim), (0, head_dim - dim))
        read = [cache_layout.read_kv(host, int(tables[s][p // page_size]), p % page_size, head_dim) for p in range(n)]
        torch.testing.assert_close(torch.stack([k for k, _ in read]).double(), keys, **t)
        torch.testing.assert_close(torch.stack([v for _, v in read]).double(), values, **t)
        if taps > 1:
            last = torch.cat([torch.zeros((taps - 1, channels), dtype=torch.float64), u])[n:]
            torch.testing.assert_close(state[slots[s]].cpu().double().reshape(taps - 1, channels), last, rtol=1e-5, atol=1e-5)
    assert taps == 1 or torch.count_nonzero(state[2]) == 0, "a slot that no sequence of the steps names was written"


# ---- routing and normalised sums ------------------------------------------------------------------------------------ #
@pytest.mark.parametrize("experts,top,groups", [(6, 3, (3, 2)), (16, 4, (4, 2)), (8, 1, (8, 1)), (256, 16, (32, 5)), (120, 8, (2, 1)), (9, 9, (3, 3)), (70, 5, None)])
def test_routes_to_the_best_groups(experts, top, groups):
    from cwm_amd import ops

    logits = rnd((37, experts), experts, 2.0)
    spec = {"count": groups[0], "keep": groups[1]} if groups else None
    chosen, weights = sp.route(logits.double(), top, spec)
    got_chosen, got_weights = ops.route_top(logits.to(DEV), top, "softmax_all", groups=groups)
    assert torch.equal(got_chosen.cpu().long(), chosen)
    torch.testing.assert_close(got_weights.cpu().double(), weights, rtol=1e-5, atol=1e-7)
    with pytest.raises(ops.KernelError):
        ops.route_top(logits.to(DEV), top, "softmax_all", groups=(experts + 1, 1))


@pytest.mark.parametrize("out_dtype", DTYPES)
@pytest.mark.parametrize("dim,top", [(192, 3), (50, 5), (2048, 4), (40, 1)])
def test_a_normalised_sum_of_routed_rows(out_dtype, dim, top):
    """The norm that adds up a token's routed rows, norms the sum, joins it to the residual and norms that: the same as the
    sum made first."""
    from cwm_amd import ops

    n, experts = 23, 7
    chosen = torch.stack([torch.randperm(experts, generator=torch.Generator().manual_seed(i))[:top] for i in range(n)]).to(torch.int32)
    groups = ops.group_by_expert(chosen.to(DEV), experts)
    rows, weights = rnd((groups.n_tiles * 16, dim), 3).to(DEV), rnd((n, top), 4).abs().to(DEV)
    h, w1, w2 = rnd((n, dim), 5), rnd((dim,), 6).to(DEV), rnd((dim,), 7).to(DEV)
    routed = ops.RoutedSum(rows, groups, weights)
    want = h.double() + sp.unit_rms(routed.combine().cpu().double(), 1e-5) * w1.cpu().double()
    got_h = h.to(DEV)
    out = ops.add_normed_rmsnorm(got_h, ops.NormedSum([(routed, w1, 1.0)], 1e-5), w2, 1e-5, out_dtype)
    torch.testing.assert_close(got_h.cpu().double(), want, rtol=1e-5, atol=1e-5)
    t = dict(rtol=1e-4, atol=1e-4) if out_dtype == torch.float32 else dict(rtol=1e-2, atol=1e-2)
    torch.testing.assert_close(out.cpu().double(), sp.unit_rms(want, 1e-5) * w2.cpu().double(), **t)
    pick = torch.tensor([20, 3], dtype=torch.int32, device=DEV)
    left = h.to(DEV)
    some = ops.add_normed_rmsnorm(left, ops.NormedSum([(routed, w1, 1.0)], 1e-5), w2, 1e-5, out_dtype, rows=pick)
    assert torch.equal(some, out[pick.long()]) and torch.equal(left.cpu(), h)


@pytest.mark.parametrize("dtype", DTYPES)
def test_gelu_gates(dtype):
    from cwm_amd import ops

    hidden, n = 48, 9
    x = rnd((n, 2 * hidden), 1, 3.0).to(dtype)
    want = sp.gelu_tanh(x[:, :hidden].double()) * x[:, hidden:].double()
    t = dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=1e-2)
    torch.testing.assert_close(ops.gated_act_rows(x.to(DEV), hidden, ops.GatedActivation("gelu_tanh"), dtype).cpu().double(), want, **t)
    # in the epilogue of the experts' product
    experts, rows = 3, rnd((n, 40), 2).to(dtype)
    gate, up = rnd((experts, hidden, 40), 3, 0.2).to(dtype), rnd((experts, hidden, 40), 4, 0.2).to(dtype)
    chosen = torch.arange(n, dtype=torch.int32)[:, None] % experts
    groups = ops.group_by_expert(chosen.to(DEV), experts)
    got = ops.grouped_gate_up(rows.to(DEV), groups, gate.to(DEV), up.to(DEV), ops.GatedActivation("gelu_tanh")).cpu()
    for i in range(n):
        e = int(chosen[i, 0])
        one = sp.gelu_tanh(rows[i].double() @ gate[e].double().T) * (rows[i].double() @ up[e].double().T)
        torch.testing.assert_close(got[int(groups.pair_row[i])].double(), one, **dict(t, atol=3e-2 if dtype == torch.bfloat16 else 1e-5))


# ---- models ---------------------------------------------------------------------------------------------------------- #
LENGTHS = {"tiny_l": [40, 75, 33, 64, 9], "tiny_m": [43, 64, 50, 7], "tiny_n": [130, 20, 66], "long": [90, 30, 7]}
PAGE_SIZES = {"whole": 16, "tail": 8, "portions": 16, "mixed": 8}


def requests_for(name, lengths=None):
    vocab = sorovik.get(name)["vocab"]
    return {f"r{i}": traces.random_tokens(17 * i + len(name), n, vocab) for i, n in enumerate(lengths or LENGTHS[name])}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("sorovik")
    return {name: sorovik.make_folder(root, name, seed=5) for name in sorovik.ALL}


@pytest.fixture(scope="module")
def plain_cache():
    return {}


def plain_for(folders, cache, name, dtype):
    if (name, dtype) not in cache:
        cache[name, dtype] = sorovik.expected(folders[name], requests_for(name), dtype, conditioning=True)
    return cache[name, dtype]


def run(folder, dtype, steps, requests, vocab, **options):
    from cwm_amd.replay import Replayer

    rep = Replayer(folder, dtype, traces.max_live_tokens(steps), poison_freed_pages=True, **options)
    page_use = traces.PageUse(rep.manager)
    outputs = traces.run_in_process(rep, steps, page_use)
    assert rep.manager.live_requests() == []
    return traces.gather(steps, outputs, {k: len(v) for k, v in requests.items()}, vocab), rep, page_use


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(sorovik.ALL))
@pytest.mark.parametrize("regime", ["whole", "tail", "portions", "mixed"])
def test_replay_regimes(folders, plain_cache, name, dtype, regime):
    requests = requests_for(name)
    vocab = sorovik.get(name)["vocab"]
    steps = {"whole": traces.whole, "tail": traces.tail_one_by_one, "portions": traces.portions,
             "mixed": lambda r: traces.mixed(r, max_live=3)}[regime](requests)
    got, rep, page_use = run(folders[name], dtype, steps, requests, vocab, page_size=PAGE_SIZES[regime], max_requests=3 if regime == "mixed" else 16)
    want = plain_for(folders, plain_cache, name, dtype)
    sorovik.check_together(got, want, dtype, f"{name} {dtype} {regime}")
    if regime == "mixed":
        for g in rep.manager.groups:
            assert page_use.pages_shared_between_requests(g.index) > 0, f"group {g.index}: no page served two requests"


A, L, D, M = sorovik.attention, sorovik.latent, sorovik.dense, sorovik.moe
SINGLE_LAYERS = {
    "latent_window": dict(layers=[L(3, 10, 6, 14, 12, 0.35, mask=9)]),
    "latent_every_key": dict(layers=[L(2, 12, 4, 8, 20, 0.3, mlp=D(24))]),
    "latent_window_of_one": dict(layers=[L(2, 7, 2, 5, 13, 0.4, mask=1)]),
    "latent_row_of_a_whole_tile": dict(layers=[L(4, 16, 8, 16, 24, 0.3, mask=20, base=1e6)]),
    "latent_on_the_first_layer_s_rows": dict(layers=[L(3, 10, 6, 14, 12, 0.35, mask=9), L(2, 6, 6, 7, 12, 0.4, mask=5, kv_from=0)]),
    "two_readers_with_longer_windows_than_the_writer": dict(
        layers=[A(2, 1, 8, 0.3, mask=3), L(3, 10, 4, 9, 12, 0.35, mask=4), L(2, 6, 4, 7, 12, 0.4, mask=21, kv_from=1), A(1, 1, 8, 0.3, mask=5, keep=2), L(1, 4, 4, 4, 12, 0.4, mask=12, kv_from=1)]),
    "a_reader_that_sees_every_key": dict(layers=[L(2, 8, 4, 8, 8, 0.3, mask=6), L(4, 8, 4, 8, 8, 0.3, kv_from=0)]),
    "attention_kept_tokens": dict(layers=[A(4, 2, 12, 0.3, mask=7, keep=3, rot=(60.0, 8))]),
    "attention_more_kept_tokens_than_window": dict(layers=[A(3, 1, 16, 0.3, mask=2, keep=19, rot=(60.0, 16), conv=4)]),
    "attention_without_kept_tokens_or_rotation": dict(layers=[A(3, 3, 10, 0.4, mask=11, conv=2)]),
    "attention_every_key_and_one_tap": dict(layers=[A(2, 2, 6, 0.5, rot=(50.0, 2), conv=1, mlp=D(20))]),
    "attention_without_a_convolution": dict(layers=[A(2, 1, 24, 0.3, mask=40, keep=1, rot=(1000.0, 24), conv=None)]),
    "attention_many_taps": dict(layers=[A(2, 2, 8, 0.3, mask=9, keep=8, rot=(100.0, 6), conv=9)]),
    "experts_of_the_best_groups": dict(layers=[A(1, 1, 8, 0.1, mask=2, mlp=M(12, 3, 24, groups=(4, 2)))]),
    "groups_of_one_expert": dict(layers=[L(1, 4, 2, 4, 6, 0.3, mask=3, mlp=M(7, 2, 12, groups=(7, 3)))]),
    "all_experts_chosen": dict(layers=[L(1, 4, 2, 4, 6, 0.3, mask=3, mlp=M(4, 4, 20, groups=(2, 2)))]),
    "one_expert_of_many_without_groups": dict(layers=[A(1, 1, 8, 0.1, mask=3, mlp=M(9, 1, 12))]),
    "feed_forward_carries_the_layer": dict(layers=[A(1, 1, 8, 0.1, mask=2, mlp=D(64))]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", list(SINGLE_LAYERS))
def test_single_layers(tmp_path, which, dtype):
    """One mechanism at a time between embedding and head: whole prompts against the same tokens in portions and one
    by one, and all against the plain implementation."""
    config = sorovik.model_of(**SINGLE_LAYERS[which])
    folder = sorovik.make_folder(tmp_path, which[:40], seed=2, config=config)
    requests = {f"r{i}": traces.random_tokens(i + 5, n, config["vocab"]) for i, n in enumerate([37, 5, 64])}
    want = sorovik.expected(folder, requests, dtype)
    for make in (traces.whole, traces.portions, lambda r: traces.tail_one_by_one(r, tail=20)):
        steps = make(requests)
        got, _, _ = run(folder, dtype, steps, requests, config["vocab"], page_size=8)
        sorovik.check_together(got, want, dtype, f"{which} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sharp_attention_over_long_sequences(folders, dtype):
    """The softmaxes are sharp: a token's result hangs on single keys at a window's edge and on the sequence's first
    tokens, which its layers keep.  A prompt of 700 tokens whole, in portions
    that end at, before and after page and window borders (down to one and two tokens), and with its last 150 tokens
    one by one."""
    name = "long"
    vocab = sorovik.get(name)["vocab"]
    requests = {"long": traces.random_tokens(99, 700, vocab)}
    want = sorovik.expected(folders[name], requests, dtype, conditioning=True)
    portions = lambda r: traces.portions(r, sizes=[64, 63, 65, 2, 126, 1, 31, 33, 128, 17, 11, 5, 16])  # noqa: E731
    for make in (traces.whole, portions, lambda r: traces.tail_one_by_one(r, tail=150)):
        steps = make(requests)
        got, _, _ = run(folders[name], dtype, steps, requests, vocab, page_size=32)
        sorovik.check(got["long"], want["long"], dtype, f"{name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_wider_layers_and_many_rows(tmp_path, dtype):
    """Width 256 and prompts of 600 and 300 tokens: the kernels' shapes for many rows, whole, in large portions beside
    each other, and with a tail of single tokens."""
    config = sorovik.MEDIUM
    folder = sorovik.make_folder(tmp_path, "medium", seed=9, config=config)
    vocab = config["vocab"]
    requests = {"a": traces.random_tokens(31, 600, vocab), "b": traces.random_tokens(32, 300, vocab)}
    want = sorovik.expected(folder, requests, dtype)
    side_by_side = [
        {"step": 0, "entries": [{"id": "a", "tokens": requests["a"][:290], "want": list(range(290))}, {"id": "b", "tokens": requests["b"][:270], "want": list(range(270))}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": requests["a"][290:], "want": list(range(310))}, {"id": "b", "tokens": requests["b"][270:], "want": list(range(30))}], "end": ["a", "b"]},
    ]
    for steps in (traces.whole(requests), side_by_side, traces.tail_one_by_one(requests, tail=20)):
        got, _, _ = run(folder, dtype, steps, requests, vocab, page_size=32)
        sorovik.check_together(got, want, dtype, f"medium {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_and_long_decoding(folders, dtype):
    """Every token a step of its own from an empty cache and a zero state, for 300 steps: windows pass over decoded
    tokens many times, and the kept tokens stay."""
    name = "long"
    vocab = sorovik.get(name)["vocab"]
    requests = {"a": traces.random_tokens(4, 300, vocab)}
    steps = traces.tail_one_by_one(requests, tail=299)
    got, _, _ = run(folders[name], dtype, steps, requests, vocab, page_size=16)
    sorovik.check(got["a"], sorovik.expected(folders[name], requests, dtype, conditioning=True)["a"], dtype, f"{name} {dtype} one by one")


def test_pages_and_state_slots_that_are_used_again_start_afresh(folders):
    """One slot and a pool of the longer request's size only: the second request finds the first one's states and
    cache rows (NaN in the pages in between) and must not read them."""
    name = "tiny_n"
    vocab = sorovik.get(name)["vocab"]
    a, b = traces.random_tokens(1, 60, vocab), traces.random_tokens(2, 25, vocab)
    both = [
        {"step": 0, "entries": [{"id": "a", "tokens": a, "want": [59]}], "end": ["a"]},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:10], "want": list(range(10))}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[10:], "want": list(range(15))}], "end": ["b"]},
    ]
    got, rep, _ = run(folders[name], "float32", both, {"a": a, "b": b}, vocab, page_size=8, max_requests=1)
    alone, _, _ = run(folders[name], "float32", both[1:], {"b": b}, vocab, page_size=8, max_requests=1)
    assert np.array_equal(got["b"], alone["b"])
    sorovik.check(got["b"], sorovik.expected(folders[name], {"b": b}, "float32")["b"], "float32", "second user of the slot")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_do_not_depend_on_the_rest_of_the_batch(folders, dtype):
    """A request's decoded tokens alone and beside two other requests' short portions: the same bits."""
    name = "tiny_l"
    vocab = sorovik.get(name)["vocab"]
    r = requests_for(name, [40, 64, 90])
    alone = [{"step": 0, "entries": [{"id": "r0", "tokens": r["r0"][:30], "want": [29]}], "end": []}] + [
        {"step": 1 + i, "entries": [{"id": "r0", "tokens": [r["r0"][30 + i]], "want": [0]}], "end": ["r0"] if i == 9 else []} for i in range(10)
    ]
    beside = [{"step": 0, "entries": [{"id": "r0", "tokens": r["r0"][:30], "want": [29]}], "end": []}]
    for i in range(10):
        entries = [{"id": "r1", "tokens": r["r1"][6 * i : 6 * i + 6], "want": [5]}, {"id": "r0", "tokens": [r["r0"][30 + i]], "want": [0]},
                   {"id": "r2", "tokens": r["r2"][8 * i : 8 * i + 8], "want": []}]
        beside.append({"step": 1 + i, "entries": entries, "end": ["r0", "r1", "r2"] if i == 9 else []})
    lengths = {"r0": r["r0"][:40], "r1": r["r1"][:60], "r2": r["r2"][:80]}
    got_alone, _, _ = run(folders[name], dtype, alone, {"r0": lengths["r0"]}, vocab, page_size=8)
    got_beside, _, _ = run(folders[name], dtype, beside, lengths, vocab, page_size=8)
    assert np.array_equal(got_alone["r0"][29:], got_beside["r0"][29:])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_steps_replayed_from_graphs_give_the_same_bits(folders, dtype):
    name = "tiny_m"
    vocab = sorovik.get(name)["vocab"]
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


@pytest.mark.parametrize("name", ["tiny_l", "tiny_n"])
def test_greedy_generation_through_the_engine(folders, name):
    """The engine's own entry point: scheduler, portions of 24 tokens, continuous batching, sampling kernel; then a
    cache that holds barely more than the longest request, so that requests wait for one another's pages and slots."""
    from cwm_amd.engine import Engine, GenArgs

    vocab = sorovik.get(name)["vocab"]
    prompts = [traces.random_tokens(20 + i, n, vocab) for i, n in enumerate([5, 17, 33, 64])]
    engine = Engine.from_folder(folders[name], GenArgs(use_sampling=False, max_batch=4, max_seq=2048, cache_block=16, max_prefill=24), dtype="float32")
    got = engine.generate_tokens(prompts, max_gen=12)
    for p, g in zip(prompts, got):
        assert g == sorovik.plain_greedy(folders[name], p, 12)
    small = Engine.from_folder(folders[name], GenArgs(use_sampling=False, max_batch=4, max_seq=96, cache_block=4, max_prefill=24), dtype="float32")
    assert small.generate_tokens(prompts, max_gen=12) == got


def test_command_line_and_trace_run_as_child_processes(folders, tmp_path):
    name = "tiny_l"
    vocab = sorovik.get(name)["vocab"]
    prompts = [traces.random_tokens(60 + i, n, vocab) for i, n in enumerate([6, 21])]
    path = tmp_path / "prompts.jsonl"
    path.write_text("".join(json.dumps({"id": i, "tokens": p}) + "\n" for i, p in enumerate(prompts)))
    cmd = [sys.executable, "-m", "cwm_amd.generate", f"checkpoint_dir={folders[name]}", f"prompts={path}", "dtype=float32",
           "gen_args.use_sampling=false", "gen_args.max_gen=7", "gen_args.max_seq=512", "gen_args.cache_block=16", "gen_args.max_batch=4"]
    res = subprocess.run(cmd, cwd=ROOT, capture_output=True, text=True, timeout=300)
    assert res.returncode == 0, res.stderr
    got = {rec["id"]: rec["tokens"] for rec in map(json.loads, res.stdout.strip().splitlines())}
    for i, p in enumerate(prompts):
        assert got[i] == sorovik.plain_greedy(folders[name], p, 7)

    requests = requests_for(name, [40, 75, 33])
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
        want = sorovik.expected(folders[name], requests, dtype)
        sorovik.check_together(got, want, dtype, f"trace_run {dtype}")


def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: every size, count, constant and the order of layers differ from draw to draw."""
    import random

    rng = random.Random(seed)
    width = rng.choice([32, 40, 48, 64, 72, 96, 100, 128, 136, 192, 200, 320])
    layers, writers = [], []
    for i in range(rng.randint(2, 6)):
        kind = rng.random()
        if kind < 0.2:
            mlp = None
        elif kind < 0.5:
            mlp = D(rng.choice([20, 36, 64, 100, 256]))
        else:
            count, size = rng.randint(1, 5), rng.randint(1, 4)
            keep = rng.randint(1, count)
            mlp = M(count * size, rng.randint(1, keep * size), rng.choice([8, 20, 36, 64, 96]), groups=(count, keep) if rng.random() < 0.8 else None)
        mask = rng.choice([None, 1, 2, 7, 16, 17, 40, 64, 100, 129])
        vdim, heads, dim = rng.choice([8, 12, 16, 32, 48, 64, 80]), rng.choice([1, 2, 3, 4, 6, 9]), rng.choice([8, 16, 20, 24, 32, 48, 64])
        scale = rng.choice([0.05, 0.1, 0.2]) * (64 / dim) ** 0.5
        if writers and rng.random() < 0.35:
            src = rng.choice(writers)
            m = layers[src]["mixer"]
            layers.append(L(heads, dim, m["rot_dim"], vdim, m["kv_rank"], scale, mask=mask, base=m["rot"]["base"], kv_from=src, mlp=mlp))
        elif rng.random() < 0.55:
            layers.append(L(heads, dim, rng.choice([2, 4, 8, 16, 32]), vdim, rng.choice([6, 16, 24, 40, 64, 96, 112]), scale, mask=mask, base=rng.choice([100.0, 1e4, 5e5]), mlp=mlp))
            writers.append(i)
        else:
            kv = rng.choice([1, 2, 3, 4])
            rot = (rng.choice([100.0, 1e4, 1e6]), rng.choice([d for d in (2, 4, 8, 16, 32, 64) if d <= dim])) if rng.random() < 0.8 else None
            layers.append(A(kv * rng.choice([1, 2, 3, 4]), kv, dim, scale, mask=mask, keep=rng.choice([None, 0, 1, 4, 17, 50]), rot=rot, conv=rng.choice([1, 2, 3, 4, 5]), mlp=mlp))
    return sorovik.model_of(layers, width=width, vocab=rng.randint(50, 700), eps=rng.choice([1e-5, 1e-6]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(tmp_path, seed, dtype):
    """Other models of the design: whole prompts, and a mixed schedule with pages of another size, against the plain
    implementation."""
    config = random_config(seed)
    folder = sorovik.make_folder(tmp_path, f"random{seed}", seed=seed, config=config)
    vocab = config["vocab"]
    requests = {f"r{i}": traces.random_tokens(7 * seed + i, n, vocab) for i, n in enumerate([3, 150, 45, 88])}
    want = sorovik.expected(folder, requests, dtype, conditioning=True)
    for steps, page in ((traces.whole(requests), 16), (traces.mixed(requests, max_live=3), 32 if seed % 2 else 8)):
        got, _, _ = run(folder, dtype, steps, requests, vocab, page_size=page, max_requests=4)
        sorovik.check_together(got, want, dtype, f"random configuration {seed} {dtype}: {json.dumps(config)}")
