"""Sunusun without a GPU: the plain implementation's mechanisms against library routines, invariants and formulas unrolled
by hand; that a mechanism left out or a place one token off would show; the strict configuration and the plan (tensor
names, run order, shared tensors with caches of their own); and everything around the kernels (descriptor, tables, pages
and slots that are used again) with torch in the kernels' place."""

import math

import numpy as np
import pytest
import torch

from helpers import cpu_ops, sunusun, traces
from plain import sunusun_plain as sp

F = torch.float64


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=F) * scale


# ---- the plain implementation's mechanisms ---------------------------------------------------------------------- #
def test_gelu_and_silu_are_the_library_s():
    z = torch.linspace(-6, 6, 101, dtype=F)
    torch.testing.assert_close(sp.gelu_erf(z), torch.nn.functional.gelu(z))
    torch.testing.assert_close(sp.silu(z), torch.nn.functional.silu(z))


def test_positions_are_sines_at_even_places_and_cosines_at_odd_ones():
    s = sp.sinusoid(torch.tensor([0, 1, 777]), 10)
    assert s[0].tolist() == [0.0, 1.0] * 5
    for i in range(5):
        assert s[2, 2 * i] == pytest.approx(math.sin(777 * 10000.0 ** (-2 * i / 10)))
        assert s[2, 2 * i + 1] == pytest.approx(math.cos(777 * 10000.0 ** (-2 * i / 10)))
    assert sp.sinusoid(torch.tensor([3]), 7).shape == (1, 7)


def test_temperature_steps_up_after_every_so_many_positions():
    t = sp.query_temperature(torch.arange(13), 0.5, 4)
    assert (t[:3] == 1.0).all()  # position 3 is the fourth
    for p, level in ((3, 1), (6, 1), (7, 2), (10, 2), (11, 3), (12, 3)):
        assert float(t[p]) == pytest.approx(1.0 + 0.5 * math.log(level + 1))


def test_distance_bias_and_softmax_with_one_in_the_denominator():
    r1, r2 = torch.tensor([0.7, 2.0], dtype=F), torch.tensor([0.3, 0.01], dtype=F)
    at = torch.arange(5)
    b = sp.distance_bias(at, at, r1, r2)
    assert float(b[0, 4, 1]) == pytest.approx(0.7 * math.log(1.0 + 0.3 * 3)) and float(b[1, 3, 3]) == 0.0
    s = rnd((2, 5, 5), 1, 3.0)
    causal = at[None, :] <= at[:, None]
    w = sp.softmax_with_one(s, causal)
    for h in range(2):
        for i in range(5):
            e = torch.exp(s[h, i, : i + 1])
            torch.testing.assert_close(w[h, i, : i + 1], e / (1.0 + e.sum()))
            assert (w[h, i, i + 1 :] == 0).all()
    # scores far below zero leave next to nothing: the one takes all of it, without an overflow
    assert float(sp.softmax_with_one(torch.full((1, 5, 5), -900.0, dtype=F), causal).sum()) == 0.0


def test_min_gru_is_an_average_over_time():
    width, dim = 3, 4
    w = {"z": rnd((width, dim), 1), "z.b": rnd((width,), 2), "x": rnd((width, dim), 3), "x.b": rnd((width,), 4), "g": rnd((width, dim), 5), "o": torch.eye(width, dtype=F)}
    h = rnd((6, dim), 6)
    z = torch.sigmoid(h @ w["z"].T + w["z.b"])
    u = h @ w["x"].T + w["x.b"]
    c = torch.where(u < 0, 1.0 / (1.0 + torch.exp(-u)), u + 0.5)
    t = 5
    state = sum(z[s] * c[s] * torch.prod(1.0 - z[s + 1 : t + 1], dim=0) for s in range(t + 1))
    torch.testing.assert_close(sp.min_gru(w, "", h)[t], state * torch.nn.functional.silu(h[t] @ w["g"].T))
    assert (sp.candidate(torch.tensor([0.0, -1e-9], dtype=F)) - 0.5).abs().max() < 1e-9  # no jump at zero


def test_wkv_counts_the_current_token_with_its_bonus_only():
    n, heads, d, e = 5, 2, 3, 4
    r, k, v, u = rnd((n, heads, d), 1), rnd((n, heads, d), 2), rnd((n, heads, e), 3), rnd((heads, d), 4)
    decay = torch.sigmoid(rnd((n, heads, d), 5))
    o = sp.wkv_scan(r, k, v, decay, u)
    t = 4
    want = torch.zeros(heads, e, dtype=F)
    for s in range(t):
        kept = torch.prod(decay[s + 1 : t], dim=0)  # the decays strictly between the two tokens
        want += (r[t] * kept * k[s]).sum(-1, keepdim=True) * v[s]
    want += (r[t] * u * k[t]).sum(-1, keepdim=True) * v[t]
    torch.testing.assert_close(o[t], want)


def test_token_mixes_start_from_zero():
    w = {f"mu.{s}": rnd((4,), i) for i, s in enumerate("rkvgw")}
    h = rnd((3, 4), 9)
    m = sp.token_mixes(w, "", h)
    torch.testing.assert_close(m["k"][0], h[0] * (1.0 - w["mu.k"]))
    torch.testing.assert_close(m["g"][2], h[2] * (1.0 - w["mu.g"]) + h[1] * w["mu.g"])


def test_a_mechanism_left_out_or_a_lost_state_would_show():
    config = sunusun.get("tiny_j")
    w = {k: v.to(F) for k, v in sunusun.draw_weights(config, 3).items()}
    toks = traces.random_tokens(5, 60, config["vocab"])
    base = sp.forward(config, w, toks)
    size = float(base.abs().max())

    def moved(change_config=None, change_weights=None):
        c, ww = sunusun.get("tiny_j"), dict(w)
        if change_config:
            change_config(c)
        if change_weights:
            change_weights(ww)
        return float((sp.forward(c, ww, toks) - base)[-1].abs().max()) / size

    assert moved(lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=8)) > 1e-3
    assert moved(lambda c: c["layers"][4]["mixer"]["left"].pop("q_temp")) > 1e-3
    assert moved(change_weights=lambda ww: ww.update({"l1.mix.left.r1": ww["l1.mix.left.r1"] * 0})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l1.mix.left.r2": ww["l1.mix.left.r2"] * 1.1})) > 1e-4
    assert moved(change_weights=lambda ww: ww.update({"l3.mix.mu.k": ww["l3.mix.mu.k"] * 0})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l6.mix.u": ww["l6.mix.u"] * 0})) > 1e-3
    assert moved(change_weights=lambda ww: ww.update({"l1.mix.right.z.b": ww["l1.mix.right.z.b"] + 20.0})) > 1e-2
    assert moved(change_weights=lambda ww: ww.update({"l6.mix.w0": ww["l6.mix.w0"] + 20.0})) > 1e-2
    assert moved(lambda c: c.update(logit_scale=1.0)) > 1e-2


# ---- configuration and plan --------------------------------------------------------------------------------------- #
def test_config_is_strict_and_the_plan_names_the_folder_s_tensors():
    from cwm_amd.config import ConfigError, parse_config
    from cwm_amd.models.model import Model
    from cwm_amd.parts.base import PagedKVSpec, StateSpec

    for name in [*sunusun.ALL, "medium"]:
        config = sunusun.get(name) if name in sunusun.ALL else sunusun.MEDIUM
        arch, typed = parse_config(config)
        model = Model(arch.build_plan(typed))
        drawn = sunusun.draw_weights(config, 1, rank=7)
        specs = model.tensor_specs()
        assert set(n for n, s in specs.items() if not s.optional) == set(drawn)
        for n, t in drawn.items():
            assert specs[n].fits(tuple(t.shape)), n
    for change in (
        lambda c: c["layers"][1]["mixer"]["left"].update(softcap=3.0),
        lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=0),
        lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4),
        lambda c: c["layers"][1]["mixer"].pop("right"),
        lambda c: c["layers"][0].update(weights_of=9),
        lambda c: c["layers"][3].update(weights_of=0),  # the two layers name each other
        lambda c: c["layers"][5]["mixer"].update(dim=11),  # other sizes than the layer whose tensors it uses
        lambda c: c["layers"][3]["mlp"].update(kind="moe"),
        lambda c: c["layers"][3].update(type="gla"),
        lambda c: c.update(embedding={"scale": 2.0}),
    ):
        bad = sunusun.get("tiny_j")
        change(bad)
        with pytest.raises(ConfigError):
            parse_config(bad)

    arch, typed = parse_config(sunusun.get("tiny_j"))
    model = Model(arch.build_plan(typed))
    # seven layers run, four have tensors; every run has a cache and a state of its own
    assert [call.layer for call in model.run_order] == [1, 0, 0, 1, 2, 1, 3]
    assert model.cache_slots == [(0,), (1, 2), (3, 4), (5,), (6, 7), (8,), (9,)] and model.writes_cache == [True] * 7
    assert all(isinstance(model.cache_specs[i], PagedKVSpec) and model.cache_specs[i].window is None for i in (1, 3, 6))
    assert all(isinstance(model.cache_specs[i], StateSpec) for i in (0, 2, 4, 5, 7, 8, 9))
    assert model.cache_specs[1].head_dim == 32 and model.cache_specs[2].shape == (36,)
    assert len(model.tensor_specs()) == len(set(model.tensor_specs())) and not any(n.startswith(("l0.", "l2.", "l5.")) for n in model.tensor_specs())


def test_a_norm_before_a_feed_forward_that_is_not_there_may_lie_in_the_folder(tmp_path, monkeypatch):
    from cwm_amd.replay import Replayer

    cpu_ops.install(monkeypatch)
    config = sunusun.get("tiny_k")
    weights = sunusun.draw_weights(config, 3)
    weights["l0.norm2"] = torch.tensor(1.0, dtype=torch.bfloat16)
    Replayer(sunusun.make_folder(tmp_path, "extra", config=config, weights=weights), "float32", 64, device="cpu")


# ---- everything around the kernels --------------------------------------------------------------------------------- #
LENGTHS = {"tiny_j": [1, 6, 21, 40], "tiny_k": [9, 33, 2, 17, 26], "tiny_l": [70, 12, 45]}


@pytest.mark.parametrize("name", list(sunusun.ALL))
@pytest.mark.parametrize("regime", ["whole", "tail", "portions", "mixed"])
def test_regimes_against_plain(tmp_path, monkeypatch, name, regime):
    """Pages that are freed and used again, state slots that are used again, portions down to two tokens, unequal
    requests side by side: with torch in the kernels' place every difference is a fault of the descriptor, the tables,
    the slots or the plan."""
    from cwm_amd.replay import Replayer

    cpu_ops.install(monkeypatch)
    folder = sunusun.make_folder(tmp_path, name, seed=3)
    vocab = sunusun.get(name)["vocab"]
    requests = {f"r{i}": traces.random_tokens(11 * i + len(name), n, vocab) for i, n in enumerate(LENGTHS[name])}
    steps = {"whole": traces.whole, "tail": lambda r: traces.tail_one_by_one(r, tail=8), "portions": traces.portions,
             "mixed": lambda r: traces.mixed(r, max_live=2, decode_tail=5)}[regime](requests)
    rep = Replayer(folder, "float32", traces.max_live_tokens(steps), device="cpu", page_size=4 if regime == "mixed" else 16,
                   max_requests=2 if regime == "mixed" else 4, poison_freed_pages=True)
    outputs = traces.run_in_process(rep, steps)
    got = traces.gather(steps, outputs, {k: len(v) for k, v in requests.items()}, vocab)
    want = sunusun.expected(folder, requests, "float32")
    for rid in requests:
        assert not np.isnan(got[rid]).any(), f"{rid}: missing or NaN logits"
        np.testing.assert_allclose(got[rid], want[rid].exact, rtol=2e-3, atol=2e-4 * float(np.abs(want[rid].exact).max()), err_msg=f"{name} {regime} {rid}")
    assert rep.manager.live_requests() == []
    assert all(f == g.pool.num_pages for f, g in zip(rep.manager.free_pages(), rep.manager.groups))


def test_greedy_generation_through_scheduler_and_engine(tmp_path, monkeypatch):
    from cwm_amd.engine import Engine, GenArgs

    cpu_ops.install(monkeypatch)
    folder = sunusun.make_folder(tmp_path, "tiny_k", seed=6)
    vocab = sunusun.get("tiny_k")["vocab"]
    prompts = [traces.random_tokens(50 + i, n, vocab) for i, n in enumerate([5, 17, 30])]
    engine = Engine.from_folder(folder, GenArgs(use_sampling=False, max_batch=2, max_seq=64, cache_block=4, max_prefill=8), dtype="float32", device="cpu")
    for p, g in zip(prompts, engine.generate_tokens(prompts, max_gen=6)):
        assert g == sunusun.plain_greedy(folder, p, 6)
