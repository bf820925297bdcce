"""Small configurations of the Sorovik architecture with weights drawn so that every mechanism matters, the writer of
their model folders, and the plain implementation's logits for them.

Sizes differ wherever two could be equal (query and key/value heads, unrotated, rotated and value parts of a head, the
latent and what is rotated beside it, windows, kept tokens, taps, experts, groups and how many are chosen), layers come
in every order, with and without a feed-forward, and layers that read another layer's rows do so with heads, value sizes
and windows of their own."""

from __future__ import annotations

import copy
import json
import os
from typing import Dict, List, Optional

import numpy as np
import torch

from helpers import digasun
from helpers.digasun import Expected, check, check_together  # noqa: F401  (the same limits, tokens at a router's close call apart)
from plain import sorovik_plain


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, mask=None, base=100.0, kv_from=None, mlp=None, kind="latent_attention") -> dict:
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}
    if mask is not None:
        mixer["mask"] = {"size": mask}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def attention(heads, kv_heads, dim, scale, mask=None, keep=None, rot=None, conv=3, mlp=None, kind="attention") -> dict:
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "conv": conv}
    if mask is not None:
        mixer["mask"] = {"size": mask} if keep is None else {"size": mask, "keep_first": keep}
    if rot is not None:  # (base, dims)
        mixer["rot"] = {"base": rot[0], "dims": rot[1]}
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int, groups: Optional[tuple] = None) -> dict:
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "router": router, "expert": {"ff": ff}}


def model_of(layers, width=40, vocab=83, eps=1e-5) -> dict:
    return {"architecture": "Sorovik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}


# a cached row of 18 elements in one of 32; a reader with more heads, other head and value sizes and a longer window than the
# layer whose rows it reads; a window of one key beside kept ones; three of six experts from two of three groups
TINY_L = model_of(
    [
        latent(3, 10, 6, 14, 12, 0.35, mask=9, mlp=dense(52)),
        attention(4, 2, 12, 0.3, mask=7, keep=3, rot=(60.0, 8), conv=3, mlp=moe(6, 3, 20, groups=(3, 2))),
        latent(5, 8, 6, 9, 12, 0.4, mask=15, kv_from=0, mlp=moe(4, 1, 24, groups=(4, 1))),
        attention(3, 3, 8, 0.5, mask=1, keep=5, rot=(1000.0, 8), conv=2),
        latent(2, 6, 6, 7, 12, 0.5, mask=4, kv_from=0, mlp=moe(5, 2, 16), kind="latent_attention_2"),
    ],
    width=48, vocab=131, eps=1e-5,
)
# sharp: large scales, so that single keys, also those at a window's edge and the kept ones, decide a token; one head a
# mixer; no rotation; one tap; every expert chosen; a group of one expert; no layer's window equals another's
TINY_M = model_of(
    [
        attention(2, 1, 16, 1.5, mask=11, keep=2, rot=(300.0, 16), conv=4, mlp=moe(8, 2, 12, groups=(8, 3))),
        latent(1, 12, 4, 8, 20, 2.5, mask=18, base=500.0, mlp=dense(30)),
        attention(1, 1, 24, 2.0, mask=23, keep=0, conv=1, mlp=moe(3, 3, 16)),
        latent(4, 5, 8, 3, 10, 1.8, mask=32, base=50.0, mlp=moe(9, 4, 8, groups=(3, 2))),
        latent(2, 7, 8, 12, 10, 2.0, mask=6, base=50.0, kv_from=3),
        attention(4, 4, 6, 1.2, mask=40, keep=17, rot=(50.0, 2), conv=7, mlp=dense(24), kind="attention_5"),
    ],
    width=40, vocab=97, eps=1e-6,
)
# heads of 80 and rows of 64 + 16; windows and kept tokens of two pages and more; every latent layer reads the first one's rows
TINY_N = model_of(
    [
        latent(2, 24, 16, 40, 64, 0.15, mask=50, base=10000.0, mlp=dense(96)),
        attention(2, 1, 80, 0.11, mask=33, keep=20, rot=(10000.0, 40), conv=4, mlp=moe(6, 2, 32, groups=(2, 1))),
        latent(6, 16, 16, 20, 64, 0.2, mask=64, base=10000.0, kv_from=0, mlp=moe(6, 4, 16, groups=(2, 2))),
        latent(1, 32, 16, 48, 64, 0.15, mask=20, base=10000.0, kv_from=0),
    ],
    width=64, vocab=211, eps=1e-5,
)
# no routers, whose close calls a comparison in bfloat16 would have to leave out: for long sequences
LONG = model_of(
    [
        attention(3, 1, 20, 0.9, mask=13, keep=4, rot=(200.0, 12), conv=4, mlp=dense(44)),
        latent(3, 14, 10, 6, 22, 0.8, mask=21, base=300.0),
        latent(2, 9, 10, 11, 22, 0.7, mask=47, base=300.0, kv_from=1, mlp=dense(36)),
        attention(4, 2, 8, 0.8, mask=29, keep=11, rot=(80.0, 4), conv=2),
    ],
    width=56, vocab=103, eps=1e-5,
)
# wider, so that prompts of some hundred tokens take the kernels' shapes for many rows
MEDIUM = model_of(
    [
        latent(8, 48, 32, 64, 96, 0.11, mask=100, base=10000.0, mlp=dense(512)),
        attention(8, 2, 64, 0.125, mask=120, keep=40, rot=(10000.0, 32), conv=4, mlp=moe(8, 2, 128, groups=(4, 2))),
        latent(4, 64, 32, 48, 96, 0.1, mask=257, base=10000.0, kv_from=0, mlp=moe(6, 3, 80, groups=(3, 2))),
        attention(4, 4, 128, 0.09, mask=64, keep=9, rot=(500000.0, 64), conv=3, mlp=dense(384)),
    ],
    width=192, vocab=320, eps=1e-5,
)

ALL = {"tiny_l": TINY_L, "tiny_m": TINY_M, "tiny_n": TINY_N, "long": LONG}


def get(name: str) -> dict:
    return copy.deepcopy(ALL[name])


def draw_weights(config: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors by name.  Matrices N(0, 1 / fan-in); norm weights around one; sinks of the size of a score; taps
    that count as much as the newest one; gates on both sides of a half; routers whose logits lie well apart."""
    gen = torch.Generator().manual_seed(seed)
    normal = lambda *shape, std=1.0: torch.randn(*shape, generator=gen) * std  # noqa: E731
    uniform = lambda lo, hi, *shape: torch.rand(*shape, generator=gen) * (hi - lo) + lo  # noqa: E731
    matrix = lambda out, inp: normal(out, inp, std=inp ** -0.5)  # noqa: E731
    width, vocab = config["width"], config["vocab"]
    w = {"embed": normal(vocab, width, std=0.7), "embed.norm": uniform(0.5, 1.5, width), "head": matrix(vocab, width) * 2.0, "final.norm": uniform(0.5, 1.5, width)}

    def expert(p: str, ff: int) -> None:
        w[p + "gate"], w[p + "up"], w[p + "down"] = matrix(ff, width) * 1.5, matrix(ff, width) * 1.5, matrix(width, ff)

    for i, layer in enumerate(config["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}.", layer["mlp"]
        q = p + "mix."
        w[p + "norm1"], w[p + "norm1b"] = uniform(0.5, 1.5, width), uniform(0.5, 1.5, width)
        if sorovik_plain.layer_kind(layer) == "latent_attention":
            heads = m["heads"]
            w[q + "q"] = matrix(heads * (m["dim"] + m["rot_dim"]), width)
            if m.get("kv_from") is None:
                w[q + "dkv"], w[q + "dkv.norm"] = matrix(m["kv_rank"] + m["rot_dim"], width), uniform(0.5, 1.5, m["kv_rank"])
            w[q + "uk"], w[q + "uv"] = matrix(heads * m["dim"], m["kv_rank"]), matrix(heads * m["vdim"], m["kv_rank"])
            w[q + "sink"], w[q + "o"] = normal(heads), matrix(width, heads * m["vdim"])
        else:
            for r, heads in (("q", m["heads"]), ("k", m["kv_heads"])):
                out = heads * m["dim"]
                w[q + r], w[q + r + ".b"], w[q + r + ".norm"] = matrix(out, width), normal(out, std=0.3), uniform(0.5, 1.5, out)
                if m.get("conv") is not None:
                    w[q + r + ".conv"] = normal(out, m["conv"], std=0.7)
            w[q + "g"], w[q + "o"] = matrix(m["heads"], width) * 2.0, matrix(width, m["heads"] * m["dim"])
        if mlp is not None:
            w[p + "norm2"], w[p + "norm2b"] = uniform(0.5, 1.5, width), uniform(0.5, 1.5, width)
            if mlp["kind"] == "dense":
                expert(p + "mlp.", mlp["ff"])
            else:
                w[p + "mlp.router"] = normal(mlp["router"]["experts"], width, std=0.3)
                for e in range(mlp["router"]["experts"]):
                    expert(p + f"mlp.e{e}.", mlp["expert"]["ff"])
    return {k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}


def make_folder(root, name: str, seed: int = 1, config: Optional[dict] = None, weights: Optional[Dict[str, torch.Tensor]] = None) -> str:
    from safetensors.torch import save_file

    config = config or get(name)
    folder = os.path.join(str(root), f"{name}_{seed}")
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(config, fh)
    save_file(weights if weights is not None else draw_weights(config, seed), os.path.join(folder, "model.safetensors"))
    return folder


read_folder = digasun.read_folder


def expected(folder: str, requests: Dict[str, List[int]], dtype: str, conditioning: bool = False) -> Dict[str, Expected]:
    config, weights = read_folder(folder)
    gen = torch.Generator().manual_seed(1)
    out = {}
    for rid, toks in requests.items():
        margins: list = []
        exact64 = sorovik_plain.forward(config, weights, toks, margins=margins)
        least = torch.stack(margins).min(0).values.numpy() if margins else np.full(len(toks), np.inf)
        rounded = loose = None
        if dtype == "bfloat16":
            rounded = sorovik_plain.forward(config, weights, toks, rounded=True).to(torch.float32).numpy()
        elif conditioning:
            shaken = [{k: v * (1.0 + 1e-7 * torch.randn(v.shape, generator=gen, dtype=torch.float64)) for k, v in weights.items()} for _ in range(2)]
            loose = np.maximum(*[(sorovik_plain.forward(config, s, toks) - exact64).abs().max(dim=1).values.numpy() for s in shaken])
            # and by the angles' rounding to float32, which at far positions is more than a sum's last bits
            sorovik_plain.ANGLES = torch.float32
            try:
                turned = (sorovik_plain.forward(config, weights, toks) - exact64).abs().max(dim=1).values.numpy()
            finally:
                sorovik_plain.ANGLES = torch.float64
            loose = np.maximum(loose, 2.0 * turned / digasun.LOOSE_FACTOR)
        out[rid] = Expected(exact64.to(torch.float32).numpy(), rounded, least, loose)
    return out


def plain_greedy(folder: str, prompt: List[int], n_new: int) -> List[int]:
    config, weights = read_folder(folder)
    toks, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(torch.argmax(sorovik_plain.forward(config, weights, toks)[-1])))
        toks.append(out[-1])
    return out
