"""The Sunusun decoder, written plainly: whole sequences, no cache, float64, one function per mechanism.
Nothing here is imported from the product; the product is compared with this.

Notation: T tokens, D the model's width.  A model is a dictionary `config` (as config.json holds it) and a
dictionary `w` of float64 tensors by the folder's names.

    x_0[p]     = E[token] + s(p),   s(p)[2i] = sin(p * 10000^(-2i/D)),  s(p)[2i + 1] = cos of the same
    layer:       x <- x + mixer(n_1(x));  x <- x + W_down gelu(W_up n_2(x))            (the second where it has an mlp)
    n(v)       = v / sqrt(mean(v^2) + eps) * g        one number g; a layer may use another layer's tensors
    parallel:    (rms(L(h)) * a + rms(R(h)) * b) / 2   over the width, a and b plain weights
      L:         q, k per head over rms times a weight;  q <- q (1 + c ln(floor((p + 1) / e) + 1));
                 s_ij = scale q_i.k_j - r1_h ln(1 + r2_h (i - j)),  j <= i;   p_ij = exp(s_ij) / (1 + sum_j exp(s_ij))
      R:         z = sigmoid(W_z h + b_z), u = W_x h + b_x;  S_t = (1 - z) S_(t-1) + z g(u);  W_o (S_t silu(W_g h))
                 g(u) = u + 1/2 for u >= 0, sigmoid(u) below
    wkv:         m_s = h_t + (h_(t-1) - h_t) mu_s for s in r, k, v, g, w;  r, k, v = W m;  d = exp(-exp(W_w2 tanh(W_w1 m_w) + w_0));
                 o_t = S_(t-1)^T r_t + (sum_c r_c u_c k_c) v_t;  S_t = diag(d_t) S_(t-1) + k_t v_t^T;
                 W_o (o over rms per head, times n, times silu(W_g m_g))
    logits     = c W_head n_final(x)
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F = torch.float64


def bf16_round(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).to(torch.bfloat16).to(t.dtype)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_erf(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def sinusoid(positions: torch.Tensor, width: int) -> torch.Tensor:
    out = torch.zeros(positions.numel(), width, dtype=F)
    for d in range(width):
        angle = positions.to(F) * 10000.0 ** (-2.0 * (d // 2) / width)
        out[:, d] = torch.sin(angle) if d % 2 == 0 else torch.cos(angle)
    return out


def query_temperature(positions: torch.Tensor, coef: float, every: float) -> torch.Tensor:
    return 1.0 + coef * torch.log(torch.floor((positions.to(F) + 1.0) / every) + 1.0)


def distance_bias(queries: torch.Tensor, keys: torch.Tensor, r1: torch.Tensor, r2: torch.Tensor) -> torch.Tensor:
    """[H, queries, keys]: what comes off the score of the query at one position and the key at another (zero where the key
    comes after the query, which nothing reads)."""
    d = (queries[:, None] - keys[None, :]).clamp(min=0).to(F)
    return r1[:, None, None] * torch.log(1.0 + r2[:, None, None] * d[None])


def softmax_with_one(scores: torch.Tensor, visible: torch.Tensor) -> torch.Tensor:
    """scores [H, queries, keys] -> exp(s) / (1 + sum exp(s)) over the visible keys of each query."""
    s = scores.masked_fill(~visible[None], float("-inf"))
    m = s.max(dim=-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(dim=-1, keepdim=True))


def attention(w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, eps: float, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    n, heads, groups, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms((rd(h @ w[p + "q"].T)).reshape(n, heads, dim), eps) * w[p + "q.norm"]
    k = rd(unit_rms((rd(h @ w[p + "k"].T)).reshape(n, groups, dim), eps) * w[p + "k.norm"])
    v = rd(h @ w[p + "v"].T).reshape(n, groups, vdim)
    if m.get("q_temp") is not None:
        q = q * query_temperature(torch.arange(n), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    q = rd(q)
    per = heads // groups
    k, v = k.repeat_interleave(per, dim=1), v.repeat_interleave(per, dim=1)
    at = torch.arange(n)
    scores = torch.einsum("ihd,jhd->hij", q, k) * m["scale"] - distance_bias(at, at, w[p + "r1"], w[p + "r2"])
    out = torch.einsum("hij,jhd->ihd", rd(softmax_with_one(scores, at[None, :] <= at[:, None])), v).reshape(n, heads * vdim)
    return rd(out) @ w[p + "o"].T


def candidate(u: torch.Tensor) -> torch.Tensor:
    return torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def min_gru(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    z = torch.sigmoid(rd(h @ w[p + "z"].T) + w[p + "z.b"])
    c = candidate(rd(h @ w[p + "x"].T) + w[p + "x.b"])
    gate = silu(rd(h @ w[p + "g"].T))
    state = torch.zeros_like(z[0])
    rows = []
    for t in range(h.shape[0]):
        state = (1.0 - z[t]) * state + z[t] * c[t]
        rows.append(state)
    return rd(torch.stack(rows) * gate) @ w[p + "o"].T


def parallel(w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, eps: float, rounded: bool = False) -> torch.Tensor:
    left = attention(w, p + "left.", m["left"], h, eps, rounded)
    right = min_gru(w, p + "right.", h, rounded)
    if rounded:
        left, right = bf16_round(left), bf16_round(right)
    return 0.5 * (unit_rms(left, eps) * w[p + "left.out"] + unit_rms(right, eps) * w[p + "right.out"])


def token_mixes(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor) -> Dict[str, torch.Tensor]:
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return {s: h + (before - h) * w[p + "mu." + s] for s in "rkvgw"}


def wkv_scan(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, u: torch.Tensor) -> torch.Tensor:
    """r, k, decay [T, H, d], v [T, H, e], u [H, d] -> o [T, H, e]."""
    n, heads, dim = r.shape
    out = torch.zeros(n, heads, v.shape[2], dtype=F)
    for head in range(heads):
        state = torch.zeros(dim, v.shape[2], dtype=F)
        for t in range(n):
            kv = k[t, head][:, None] * v[t, head][None, :]
            out[t, head] = (state + u[head][:, None] * kv).T @ r[t, head]
            state = decay[t, head][:, None] * state + kv
    return out


def wkv(w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, eps: float, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    n, heads, dim = h.shape[0], m["heads"], m["dim"]
    mix = {s: rd(t) for s, t in token_mixes(w, p, h).items()}
    r, k, v = (rd(mix[s] @ w[p + s].T).reshape(n, heads, dim) for s in "rkv")
    gate = silu(rd(mix["g"] @ w[p + "g"].T))
    low = torch.tanh(mix["w"] @ w[p + "w1"].T)
    decay = torch.exp(-torch.exp(low @ w[p + "w2"].T + w[p + "w0"])).reshape(n, heads, dim)
    o = wkv_scan(r, k, v, decay, w[p + "u"])
    return rd(unit_rms(o, eps).reshape(n, heads * dim) * w[p + "norm"] * gate) @ w[p + "o"].T


def feed_forward(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    return rd(gelu_erf(h @ w[p + "up"].T)) @ w[p + "down"].T


def owner(config: dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while config["layers"][i].get("weights_of") is not None:
        i = config["layers"][i]["weights_of"]
    return i


def forward(config: dict, w: Dict[str, torch.Tensor], tokens: List[int], rounded: bool = False, layers: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  `rounded`: as a run in bfloat16 stores what lies between the kernels.
    `layers` receives the residual after every layer."""
    rd = bf16_round if rounded else (lambda t: t)
    eps = config["norm"]["eps"]
    norm = lambda name, x, gain=1.0: rd(unit_rms(x, eps) * (w[name] * gain))  # noqa: E731
    x = w["embed"][tokens] + sinusoid(torch.arange(len(tokens)), config["width"])
    for i, layer in enumerate(config["layers"]):
        p = f"l{owner(config, i)}."
        h = norm(p + "norm1", x)
        if layer["type"].split("_")[0] == "parallel":
            x = x + parallel(w, p + "mix.", layer["mixer"], h, eps, rounded)
        else:
            x = x + wkv(w, p + "mix.", layer["mixer"], h, eps, rounded)
        if layer["mlp"] is not None:
            x = x + feed_forward(w, p + "mlp.", norm(p + "norm2", x), rounded)
        if layers is not None:
            layers.append(x.clone())
    return norm("final.norm", x, config["logit_scale"]) @ w["head"].T
