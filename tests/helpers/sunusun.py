"""Small configurations of the Sunusun architecture with weights drawn so that every mechanism matters, the writer of
their model folders, and the plain implementation's logits for them.

Sizes differ wherever two could be equal (query and key/value heads, query/key and value head sizes, the recurrence's
width and the model's, the heads of the two kinds of mixer, the feed-forwards); layers come in every order, with and
without a feed-forward, with tensors of their own or of an earlier or a later layer."""

from __future__ import annotations

import copy
import json
import os
from typing import Dict, List, Optional

import numpy as np
import torch

from helpers import lapevik  # the same limits: float32 sums in another order; what bfloat16 storage costs
from plain import sunusun_plain


def parallel(heads, kv_heads, dim, vdim, scale, width, temp=None, mlp=None, weights_of=None, kind="parallel") -> dict:
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if temp is not None:  # (coef, every)
        left["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return _layer(kind, {"left": left, "right": {"width": width}}, mlp, weights_of)


def wkv(heads, dim, mlp=None, weights_of=None, kind="wkv") -> dict:
    return _layer(kind, {"heads": heads, "dim": dim}, mlp, weights_of)


def _layer(kind, mixer, mlp, weights_of) -> dict:
    layer = {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": mlp} if mlp is not None else None}
    if weights_of is not None:
        layer["weights_of"] = weights_of
    return layer


def model_of(layers, width=40, vocab=83, eps=1e-5, logit_scale=1.5) -> dict:
    layers = [dict(copy.deepcopy(layer)) for layer in layers]
    for layer in layers:
        j = layer.get("weights_of")
        if j is not None:  # the rest of such an entry repeats the other layer's
            layer["mixer"], layer["mlp"] = copy.deepcopy(layers[j]["mixer"]), copy.deepcopy(layers[j]["mlp"])
    return {"architecture": "Sunusun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


# heads of 12 and 20 share a cached head of 32; a layer that runs three times with one set of tensors, once before the layer
# that has them; a layer without a feed-forward
TINY_J = model_of(
    [
        wkv(0, 0, weights_of=3),
        parallel(6, 2, 12, 20, 0.3, 36, temp=(0.5, 7), mlp=56),
        parallel(0, 0, 0, 0, 0, 0, weights_of=1),
        wkv(3, 10, mlp=44),
        parallel(2, 2, 16, 8, 0.4, 52, temp=(0.2, 3), kind="parallel_2"),
        wkv(0, 0, weights_of=3),
        wkv(2, 17, kind="wkv_5"),
    ],
    width=48, vocab=131, logit_scale=1.7,
)
# sharp: large scales, so that single keys decide a token; one head a mixer; queries that grow with every token, and a
# layer whose queries do not; the first layer and the last end without a feed-forward
TINY_K = model_of(
    [
        parallel(2, 1, 16, 10, 1.5, 21, temp=(0.1, 1)),
        wkv(1, 33, mlp=30),
        parallel(4, 4, 8, 8, 2.0, 40, mlp=24),
        wkv(4, 6, mlp=20),
        parallel(3, 1, 20, 33, 1.0, 8, temp=(-0.1, 50), kind="parallel_9"),
    ],
    width=40, vocab=97, eps=1e-6, logit_scale=0.6,
)
# heads of 80; a state whose rows are shared by lanes; steps of the temperature at a page's size
TINY_L = model_of(
    [
        parallel(2, 1, 80, 48, 0.11, 100, temp=(0.4, 16), mlp=96),
        wkv(2, 40, mlp=72),
        wkv(1, 72, mlp=64),
        parallel(0, 0, 0, 0, 0, 0, weights_of=0),
    ],
    width=64, vocab=211, logit_scale=3.0,
)
# wider, so that prompts of some hundred tokens take the kernels' shapes for many rows
MEDIUM = model_of(
    [
        parallel(8, 2, 64, 64, 0.125, 224, temp=(0.25, 100), mlp=512),
        wkv(4, 64, mlp=384),
        wkv(2, 128, mlp=320),
        parallel(4, 4, 128, 64, 0.09, 96, temp=(0.3, 64), mlp=448),
    ],
    width=192, vocab=320, logit_scale=1.2,
)

ALL = {"tiny_j": TINY_J, "tiny_k": TINY_K, "tiny_l": TINY_L}


def get(name: str) -> dict:
    return copy.deepcopy(ALL[name])


def layer_kind(layer: dict) -> str:
    return layer["type"].split("_")[0]


def draw_weights(config: dict, seed: int, rank: int = 5) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors by name.  Matrices N(0, 1 / fan-in); norm weights around one; distance biases that leave far keys
    a share; gates and decays between those that forget within a token and those that keep a state for hundreds."""
    gen = torch.Generator().manual_seed(seed)
    normal = lambda *shape, std=1.0: torch.randn(shape, generator=gen) * std  # noqa: E731
    uniform = lambda lo, hi, *shape: torch.rand(shape, generator=gen) * (hi - lo) + lo  # noqa: E731
    matrix = lambda out, inp: normal(out, inp, std=inp ** -0.5)  # noqa: E731
    width, vocab = config["width"], config["vocab"]
    w = {"embed": normal(vocab, width), "head": matrix(vocab, width), "final.norm": uniform(0.8, 1.4)}
    for i, layer in enumerate(config["layers"]):
        if layer.get("weights_of") is not None:
            continue
        m, p, mlp = layer["mixer"], f"l{i}.", layer["mlp"]
        w[p + "norm1"] = uniform(0.7, 1.4)
        q = p + "mix."
        if layer_kind(layer) == "parallel":
            a, r = m["left"], m["right"]["width"]
            left, right = q + "left.", q + "right."
            w[left + "q"], w[left + "k"] = matrix(a["heads"] * a["dim"], width), matrix(a["kv_heads"] * a["dim"], width)
            w[left + "v"], w[left + "o"] = matrix(a["kv_heads"] * a["vdim"], width), matrix(width, a["heads"] * a["vdim"])
            w[left + "q.norm"], w[left + "k.norm"] = uniform(0.5, 1.5, a["dim"]), uniform(0.5, 1.5, a["dim"])
            w[left + "r1"], w[left + "r2"] = uniform(0.05, 1.2, a["heads"]), uniform(0.02, 0.5, a["heads"])
            for s in "zxg":
                w[right + s] = matrix(r, width)
            w[right + "z.b"], w[right + "x.b"], w[right + "o"] = uniform(-6.0, 1.0, r), normal(r, std=0.5), matrix(width, r)
            w[left + "out"], w[right + "out"] = uniform(0.5, 1.5, width), uniform(0.5, 1.5, width)
        else:
            inner = m["heads"] * m["dim"]
            for s in "rkvgw":
                w[q + "mu." + s] = uniform(0.1, 0.9, width)
            for s in "rkvg":
                w[q + s] = matrix(inner, width)
            w[q + "w1"], w[q + "w2"], w[q + "w0"] = matrix(rank, width) * 1.5, matrix(inner, rank) * 1.5, uniform(-6.0, 0.5, inner)
            w[q + "u"], w[q + "norm"], w[q + "o"] = normal(m["heads"], m["dim"]), uniform(0.5, 1.5, inner), matrix(width, inner)
        if mlp is not None:
            w[p + "norm2"] = uniform(0.7, 1.4)
            w[p + "mlp.up"], w[p + "mlp.down"] = matrix(mlp["ff"], width) * 1.5, matrix(width, mlp["ff"])
    return {k: v.reshape(()).to(torch.bfloat16) if k.split(".")[-1] in ("norm1", "norm2") or k == "final.norm" else v.to(torch.bfloat16).contiguous() for k, v in w.items()}


def make_folder(root, name: str, seed: int = 1, config: Optional[dict] = None, weights: Optional[Dict[str, torch.Tensor]] = None) -> str:
    from safetensors.torch import save_file

    config = config or get(name)
    folder = os.path.join(str(root), f"{name}_{seed}")
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(config, fh)
    save_file(weights if weights is not None else draw_weights(config, seed), os.path.join(folder, "model.safetensors"))
    return folder


def read_folder(folder: str):
    from safetensors.torch import load_file

    with open(os.path.join(folder, "config.json")) as fh:
        config = json.load(fh)
    return config, {k: v.to(torch.float64) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}


LOOSE_FACTOR = 50.0  # float32 sums in another order, as a multiple of a change of the weights by 1e-7 of themselves


class Expected(lapevik.Expected):
    """Exact logits, what bfloat16 storage alone costs, and, for float32 runs that ask for it, how far every position's
    logits move when all weights change in their last float32 bits."""

    def __init__(self, exact: np.ndarray, rounded: Optional[np.ndarray], loose: Optional[np.ndarray] = None) -> None:
        super().__init__(exact, rounded)
        self.loose = loose


def expected(folder: str, requests: Dict[str, List[int]], dtype: str, conditioning: bool = False) -> Dict[str, Expected]:
    config, weights = read_folder(folder)
    gen = torch.Generator().manual_seed(1)
    out = {}
    for rid, toks in requests.items():
        exact64 = sunusun_plain.forward(config, weights, toks)
        rounded = loose = None
        if dtype == "bfloat16":
            rounded = sunusun_plain.forward(config, weights, toks, rounded=True).to(torch.float32).numpy()
        elif conditioning:
            shaken = {k: v * (1.0 + 1e-7 * torch.randn(v.shape, generator=gen, dtype=torch.float64)) for k, v in weights.items()}
            loose = (sunusun_plain.forward(config, shaken, toks) - exact64).abs().max(dim=1).values.numpy()
        out[rid] = Expected(exact64.to(torch.float32).numpy(), rounded, loose)
    return out


def check(got: np.ndarray, want: Expected, dtype: str, what: str) -> None:
    if dtype != "float32" or want.loose is None:
        return lapevik.check(got, want, dtype, what)
    assert got.shape == want.exact.shape and not np.isnan(got).any(), f"{what}: missing or NaN logits"
    err = np.abs(got.astype(np.float64) - want.exact.astype(np.float64)).max(axis=1)
    limit = lapevik.FLOAT32_LIMIT * float(np.abs(want.exact).max()) + LOOSE_FACTOR * want.loose
    over = err - limit
    assert over.max() <= 0, f"{what}: first position over its limit {int(np.argmax(over > 0))}, error {err[np.argmax(over)]:.3e} vs {limit[np.argmax(over)]:.3e}"


def check_together(got: Dict[str, np.ndarray], want: Dict[str, Expected], dtype: str, what: str) -> None:
    """Every request on its own in float32; in bfloat16 all requests of a model as one, since what bfloat16 storage costs
    is itself a draw, and a request of a few tokens is a small sample of it."""
    if dtype != "bfloat16":
        for rid in want:
            check(got[rid], want[rid], dtype, f"{what} {rid}")
        return
    pooled = lapevik.Expected.__new__(lapevik.Expected)
    pooled.exact = np.concatenate([want[r].exact for r in want])
    sizes = np.array([want[r].exact.size for r in want], dtype=np.float64)
    pooled.rms = float(np.sqrt((sizes * np.array([want[r].rms for r in want]) ** 2).sum() / sizes.sum()))
    pooled.max = max(want[r].max for r in want)
    lapevik.check(np.concatenate([got[r] for r in want]), pooled, dtype, what)


def plain_greedy(folder: str, prompt: List[int], n_new: int) -> List[int]:
    config, weights = read_folder(folder)
    toks, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(torch.argmax(sunusun_plain.forward(config, weights, toks)[-1])))
        toks.append(out[-1])
    return out
