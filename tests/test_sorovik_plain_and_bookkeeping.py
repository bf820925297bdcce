"""Sorovik without a GPU: the plain implementation's mechanisms against library routines, invariants and formulas
unrolled by hand; that a mechanism left out or a window one key off would show; the strict configuration and the plan
(tensor names, run order, which rows are shared, what a shared cache and a cache of kept tokens keep); and everything
around the kernels (descriptor, tables, pages and slots that are used again) with torch in the kernels' place."""

import math

import numpy as np
import pytest
import torch

from helpers import cpu_ops, sorovik, traces
from plain import sorovik_plain as sp

F = torch.float64


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=F) * scale


# ---- the plain implementation's mechanisms ---------------------------------------------------------------------- #
def test_norm_and_activations_are_the_library_s():
    x, g = rnd((5, 24), 1, 3.0), rnd((24,), 2)
    torch.testing.assert_close(sp.unit_rms(x, 1e-5) * g, torch.nn.functional.rms_norm(x, (24,), g, 1e-5))
    z = torch.linspace(-6, 6, 101, dtype=F)
    torch.testing.assert_close(sp.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    torch.testing.assert_close(sp.silu(z), torch.nn.functional.silu(z))


def test_convolution_is_the_library_s_with_zeros_before_the_start():
    u, w = rnd((11, 6), 1), rnd((6, 4), 2)
    lib = torch.nn.functional.conv1d(torch.nn.functional.pad(u.T[None], (3, 0)), w[:, None, :], groups=6)[0].T
    torch.testing.assert_close(sp.causal_conv(u, w), lib)
    only_last = torch.zeros(6, 4, dtype=F)
    only_last[:, 3] = 2.0
    torch.testing.assert_close(sp.causal_conv(u, only_last), 2.0 * u)


def test_rotation_pairs_halves_of_the_turned_part():
    x = rnd((3, 2, 10), 1)
    y = sp.turn_halves(x, torch.tensor([0, 5, 117]), 6, 100.0)
    torch.testing.assert_close(y[0], x[0])
    torch.testing.assert_close(y[..., 6:], x[..., 6:])
    for i in range(3):
        a = 117 * 100.0 ** (-2 * i / 6)
        u, v = x[2, :, i], x[2, :, i + 3]
        torch.testing.assert_close(y[2, :, i], u * math.cos(a) - v * math.sin(a))
        torch.testing.assert_close(y[2, :, i + 3], v * math.cos(a) + u * math.sin(a))
    q, k = rnd((1, 1, 6), 2), rnd((1, 1, 6), 3)
    s = lambda p, r: (sp.turn_halves(q, torch.tensor([p]), 6, 100.0) * sp.turn_halves(k, torch.tensor([r]), 6, 100.0)).sum()  # noqa: E731
    torch.testing.assert_close(s(40, 33), s(1007, 1000))


def test_windows_and_kept_first_tokens():
    seen = lambda *a: [torch.nonzero(row)[:, 0].tolist() for row in sp.visible_keys(*a)]  # noqa: E731
    assert seen(4, 2) == [[0], [0, 1], [1, 2], [2, 3]]
    assert seen(6, 2, 1) == [[0], [0, 1], [0, 1, 2], [0, 2, 3], [0, 3, 4], [0, 4, 5]]
    assert seen(5, 1, 3) == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 4]]
    assert seen(3, None) == [[0], [0, 1], [0, 1, 2]]


def test_the_sink_takes_its_share():
    scores, sink = rnd((3, 6, 6), 1), torch.tensor([0.3, -2.0, 5.0], dtype=F)
    w = sp.sink_softmax(scores, sp.visible_keys(6, 3, 1), sink)
    for h in range(3):
        e = torch.exp(scores[h, 5, [0, 3, 4, 5]])
        torch.testing.assert_close(w[h, 5, [0, 3, 4, 5]], e / (e.sum() + math.exp(float(sink[h]))))
        assert w[h, 5, 1] == 0 and w[h, 5, 2] == 0


def test_latent_attention_is_the_unrolled_formula_for_one_query():
    width, m = 16, {"heads": 3, "dim": 5, "rot_dim": 4, "vdim": 6, "kv_rank": 7, "scale": 0.37, "mask": {"size": 3}, "rot": {"base": 50.0, "dims": 4}}
    w = {"q": rnd((27, width), 1, 0.3), "dkv": rnd((11, width), 2, 0.3), "dkv.norm": rnd((7,), 3), "uk": rnd((15, 7), 4), "uv": rnd((18, 7), 5),
         "sink": rnd((3,), 6), "o": rnd((width, 18), 7)}
    h = rnd((6, width), 9)
    out = sp.latent_attention(w, "", m, h, *sp.latent_rows(w, "", m, h, 1e-5))
    heads = []
    for g in range(3):
        q = (w["q"] @ h[5]).reshape(3, 9)[g]
        scores, values = [], []
        for j in (3, 4, 5):
            down = w["dkv"] @ h[j]
            c = down[:7] / torch.sqrt((down[:7] ** 2).mean() + 1e-5) * w["dkv.norm"]
            turn = lambda x, p: sp.turn_halves(x.reshape(1, 1, 4), torch.tensor([p]), 4, 50.0).reshape(4)  # noqa: E731
            scores.append(0.37 * (q[:5] @ (w["uk"][5 * g : 5 * g + 5] @ c) + turn(q[5:], 5) @ turn(down[7:], j)))
            values.append(w["uv"][6 * g : 6 * g + 6] @ c)
        e = torch.exp(torch.stack(scores))
        heads.append(sum(x * v for x, v in zip(e / (e.sum() + torch.exp(w["sink"][g])), values)))
    torch.testing.assert_close(out[5], w["o"] @ torch.cat(heads))


def test_attention_is_the_unrolled_formula_for_one_query():
    width, m = 12, {"heads": 4, "kv_heads": 2, "dim": 6, "scale": 0.4, "conv": 3, "mask": {"size": 2, "keep_first": 1}, "rot": {"base": 50.0, "dims": 4}}
    w = {"q": rnd((24, width), 1, 0.3), "q.b": rnd((24,), 2), "q.conv": rnd((24, 3), 3), "q.norm": rnd((24,), 4), "k": rnd((12, width), 5, 0.3),
         "k.b": rnd((12,), 6), "k.conv": rnd((12, 3), 7), "k.norm": rnd((12,), 8), "g": rnd((4, width), 9), "o": rnd((width, 24), 10)}
    h = rnd((5, width), 11)
    out = sp.attention(w, "", m, h, 1e-5)

    def convolved(name, t):
        u = lambda s: w[name] @ h[s] + w[name + ".b"] if s >= 0 else torch.zeros(w[name].shape[0], dtype=F)  # noqa: E731
        return w[name + ".conv"][:, 0] * u(t - 2) + w[name + ".conv"][:, 1] * u(t - 1) + w[name + ".conv"][:, 2] * u(t)

    def ready(name, t, heads):
        y = convolved(name, t)
        y = y / torch.sqrt((y * y).mean() + 1e-5) * w[name + ".norm"]
        return sp.turn_halves(y.reshape(1, heads, 6), torch.tensor([t]), 4, 50.0)[0]

    q = ready("q", 4, 4)
    heads = []
    for g in range(4):
        e = torch.exp(torch.stack([0.4 * (q[g] @ ready("k", j, 2)[g // 2]) for j in (0, 3, 4)]))
        values = [convolved("k", j).reshape(2, 6)[g // 2] for j in (0, 3, 4)]
        heads.append(torch.sigmoid(w["g"][g] @ h[4]) * sum(x * v for x, v in zip(e / (1 + e.sum()), values)))
    torch.testing.assert_close(out[4], w["o"] @ torch.cat(heads))


def test_router_takes_the_best_experts_of_the_best_groups():
    logits = torch.tensor([[3.0, 0.0, 2.0, 1.9, 2.5, -1.0], [0.0, 0.1, 0.2, 0.3, 0.4, 0.5]], dtype=F)
    s = torch.softmax(logits, -1)
    chosen, weights = sp.route(logits, 3)
    assert chosen.tolist() == [[0, 4, 2], [5, 4, 3]]
    chosen, weights = sp.route(logits, 3, {"count": 3, "keep": 2})  # groups (0, 1), (2, 3), (4, 5): best members 3, 2, 2.5
    assert chosen.tolist() == [[0, 4, 1], [5, 4, 3]]
    torch.testing.assert_close(weights, torch.gather(s, 1, chosen))  # of the softmax over all, as they are
    margins = sp.route_margin(logits, 3, {"count": 3, "keep": 2})
    torch.testing.assert_close(margins, torch.tensor([0.5 / 3.0, 0.1 / 0.5], dtype=F))  # the second group over the third; expert 3 over expert 2
    assert torch.isinf(sp.route_margin(logits, 6, {"count": 3, "keep": 3})).all()


def test_a_mechanism_left_out_or_a_window_one_key_off_would_show():
    w = {k: v.to(F) for k, v in sorovik.draw_weights(sorovik.get("tiny_m"), 3).items()}
    toks = traces.random_tokens(5, 70, 97)
    base = sp.forward(sorovik.get("tiny_m"), w, toks)

    def moved(change_config=None, change_weights=None):
        c, ww = sorovik.get("tiny_m"), dict(w)
        if change_config:
            change_config(c)
        if change_weights:
            change_weights(ww)
        return float((sp.forward(c, ww, toks) - base).abs().max()) / float(base.abs().max())

    for i in (0, 1, 3, 4):
        size = sorovik.get("tiny_m")["layers"][i]["mixer"]["mask"]["size"]
        for other in (size - 1, size + 1):
            assert moved(lambda c: c["layers"][i]["mixer"]["mask"].update(size=other)) > 1e-2, (i, other)
    for other in (1, 3):
        assert moved(lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=other)) > 1e-2
    # (a sink scales its head's result: with one head the norm after the mixer takes that away again)
    assert moved(change_weights=lambda ww: ww.update({"l3.mix.sink": ww["l3.mix.sink"] + torch.tensor([12.0, 0.0, 0.0, 0.0], dtype=F)})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l0.mix.k.conv": ww["l0.mix.k.conv"] * torch.tensor([0.0, 1.0, 1.0, 1.0], dtype=F)})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l0.mix.g": ww["l0.mix.g"] * 0.0})) > 1e-2
    assert moved(lambda c: c["layers"][3]["mlp"]["router"]["groups"].update(keep=1 + 2)) > 1e-2
    assert moved(lambda c: c["layers"][4]["mixer"].update(kv_from=1, rot_dim=4, kv_rank=20, rot={"base": 500.0, "dims": 4}),
                 lambda ww: ww.update({"l4.mix.q": ww["l4.mix.q"][:22], "l4.mix.uk": rnd((14, 20), 1), "l4.mix.uv": rnd((24, 20), 2)})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l2.norm1b": ww["l2.norm1b"] * 0.5})) > 1e-2


# ---- configuration and plan --------------------------------------------------------------------------------------- #
def test_config_is_strict_and_the_plan_names_the_folder_s_tensors():
    from cwm_amd.config import ConfigError, parse_config
    from cwm_amd.models.model import Model
    from cwm_amd.models.sorovik import cache_windows
    from cwm_amd.parts.base import KeptFirstKVSpec, PagedKVSpec, StateSpec

    for name in sorovik.ALL:
        config = sorovik.get(name)
        arch, typed = parse_config(config)
        specs = Model(arch.build_plan(typed)).tensor_specs()
        drawn = sorovik.draw_weights(config, 1)
        assert {n for n, s in specs.items() if not s.optional} == set(drawn)
        for n, t in drawn.items():
            assert specs[n].fits(tuple(t.shape)), n
    bad = sorovik.get("tiny_l")
    bad["layers"][0]["mixer"]["softcap"] = 3.0
    with pytest.raises(ConfigError, match="softcap"):
        parse_config(bad)
    for change in (
        lambda c: c["layers"][2]["mixer"].update(kv_from=1),  # not a layer of latent attention
        lambda c: c["layers"][2]["mixer"].update(kv_from=2),  # not an earlier layer
        lambda c: c["layers"][4]["mixer"].update(kv_from=2),  # a layer without rows of its own
        lambda c: c["layers"][2]["mixer"].update(kv_rank=16),  # other sizes than the layer it reads
        lambda c: c["layers"][2]["mixer"].update(rot={"base": 99.0, "dims": 6}),
        lambda c: c["layers"][0]["mixer"].update(rot_dim=7),
        lambda c: c["layers"][1]["mixer"].update(vdim=16),  # the values are the keys
        lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1),
        lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=1),  # kept tokens are the other mixer's
        lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4),  # six experts in four groups
        lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=1),  # two experts for three choices
        lambda c: c["layers"][1].update(type="mamba"),
    ):
        bad = sorovik.get("tiny_l")
        change(bad)
        with pytest.raises(ConfigError):
            parse_config(bad)

    arch, typed = parse_config(sorovik.get("tiny_l"))
    model = Model(arch.build_plan(typed))
    # pages of rows; pages and a convolution's state; the first layer's rows again; pages and a state; the first layer's rows
    assert model.cache_slots == [(0,), (1, 2), (0,), (3, 4), (0,)]
    assert model.writes_cache == [True, True, False, True, False]
    rows, kept = model.cache_specs[0], model.cache_specs[1]
    assert isinstance(rows, PagedKVSpec) and rows.window == 15 and rows.head_dim == 32 and rows.n_kv_heads == 1  # the longest reader's window
    assert isinstance(kept, KeptFirstKVSpec) and (kept.window, kept.keep_first, kept.head_dim) == (7, 3, 16)
    assert isinstance(model.cache_specs[2], StateSpec) and model.cache_specs[2].shape == (2 * 6 * 12,)
    assert kept.pinned_keys() == 3 and kept.first_key_needed(20) == 14 and kept.retention() != rows.retention()
    wide = sorovik.model_of([sorovik.latent(2, 8, 4, 8, 8, 0.3, mask=6), sorovik.latent(4, 8, 4, 8, 8, 0.3, kv_from=0)])
    assert cache_windows(parse_config(wide)[1]) == {0: None}


def test_a_convolution_of_one_tap_or_none_keeps_no_state():
    from cwm_amd.config import parse_config
    from cwm_amd.models.model import Model

    for conv in (1, None):
        arch, typed = parse_config(sorovik.model_of([sorovik.attention(2, 1, 8, 0.3, mask=4, conv=conv)]))
        model = Model(arch.build_plan(typed))
        assert len(model.cache_specs) == 1
        assert ("l0.mix.q.conv" in model.tensor_specs()) == (conv is not None)


def test_pages_of_kept_tokens_stay_and_pages_between_go_back():
    from cwm_amd.cache import CacheManager
    from cwm_amd.parts.base import KeptFirstKVSpec

    manager = CacheManager([KeptFirstKVSpec(1, 16, window=6, keep_first=5)], page_size=4, num_pages=8, max_requests=2)
    manager.admit("a")
    gone = []
    for _ in range(30):
        assert manager.extend("a", 1)
        gone += manager.advance("a", 1)[0]
        manager.check()
    table = manager.table(0, "a")
    assert table[0] >= 0 and table[1] >= 0  # keys 0..4 lie in the first two pages
    # the next query, at 30, reads keys 25..30: pages 2..5 (keys 8..23) have gone back, and pages were used again
    assert table[2:6] == [-1] * 4 and table[6] >= 0 and len(gone) == 4 and manager.pages_held("a") == [4]
    manager.release("a")
    assert manager.free_pages() == [8]


# ---- everything around the kernels --------------------------------------------------------------------------------- #
LENGTHS = {"tiny_l": [1, 6, 21, 40], "tiny_m": [9, 33, 2, 17, 26], "tiny_n": [70, 12, 45], "long": [50, 3, 31]}


@pytest.mark.parametrize("name", list(sorovik.ALL))
@pytest.mark.parametrize("regime", ["whole", "tail", "portions", "mixed"])
def test_regimes_against_plain(tmp_path, monkeypatch, name, regime):
    """Pages that are freed (by windows, the shared cache and the one with kept tokens among them) and used again, state
    slots that are used again, portions down to two tokens, unequal requests side by side: with torch in the kernels' place
    every difference is a fault of the descriptor, the tables, the slots or the plan."""
    from cwm_amd.replay import Replayer

    cpu_ops.install(monkeypatch)
    folder = sorovik.make_folder(tmp_path, name, seed=3)
    vocab = sorovik.get(name)["vocab"]
    requests = {f"r{i}": traces.random_tokens(11 * i + len(name), n, vocab) for i, n in enumerate(LENGTHS[name])}
    steps = {"whole": traces.whole, "tail": lambda r: traces.tail_one_by_one(r, tail=8), "portions": traces.portions,
             "mixed": lambda r: traces.mixed(r, max_live=2, decode_tail=5)}[regime](requests)
    rep = Replayer(folder, "float32", traces.max_live_tokens(steps), device="cpu", page_size=4 if regime == "mixed" else 16,
                   max_requests=2 if regime == "mixed" else 4, poison_freed_pages=True)
    outputs = traces.run_in_process(rep, steps)
    got = traces.gather(steps, outputs, {k: len(v) for k, v in requests.items()}, vocab)
    want = sorovik.expected(folder, requests, "float32")
    for rid in requests:
        assert not np.isnan(got[rid]).any(), f"{rid}: missing or NaN logits"
        np.testing.assert_allclose(got[rid], want[rid].exact, rtol=2e-3, atol=2e-4 * float(np.abs(want[rid].exact).max()), err_msg=f"{name} {regime} {rid}")
    assert rep.manager.live_requests() == []
    assert all(f == g.pool.num_pages for f, g in zip(rep.manager.free_pages(), rep.manager.groups))
