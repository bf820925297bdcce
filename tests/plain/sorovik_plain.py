"""The Sorovik decoder, written plainly: whole sequences, no cache, float64, one function per mechanism.
Nothing here is imported from the product; the product is compared with this.

Notation: T tokens, D the model's width.  A model is a dictionary `config` (as config.json holds it) and a
dictionary `w` of float64 tensors by the folder's names.

    n(v; g)    = v / sqrt(mean(v^2) + eps) * g
    x_0        = n(E[token]; embed.norm)
    layer:       x <- x + n(mixer(n(x; norm1)); norm1b);   x <- x + n(ff(n(x; norm2)); norm2b)     (the second where it has an mlp)
    latent:      q_h = (W_q h)_h = [a_h | r_h];  [c | k'] = W_dkv h,  c <- n(c; dkv.norm);  r_h, k' turned by their positions;
                 s_h(i, j) = scale (a_h,i . W_uk,h c_j + r_h,i . k'_j)   over 0 <= i - j < size;
                 p = exp(s) / (exp(sink_h) + sum exp(s));   W_o [sum_j p_ij W_uv,h c_j of every head]
                 with `kv_from` c and k' are another layer's
    attention:   u = W h + b for q and k;  y_t = sum over lags of w[:, taps - 1 - lag] u_(t - lag);  v = y of k;
                 q, k = n(y; q.norm / k.norm) over all heads at once, turned by their positions;
                 s = scale q_i . k_j   over j <= i with i - j < size or j < keep_first;   p = exp(s) / (1 + sum exp(s));
                 W_o [sigmoid(W_g h)_h * sum_j p_ij v_j of every head]
    turned:      of the first `dims` elements of a head, (e, e + dims/2) turned by p * base^(-2e/dims)
    dense ff:    W_down (gelu_tanh(W_gate h) * W_up h)
    experts:     s = softmax(W_r h);  the groups (neighbours) with the largest best score stay;  of their experts the `top` largest s;
                 sum_e s_e W_down,e (silu(W_gate,e h) * W_up,e h)
    logits     = W_head n(x; final.norm)
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

F = torch.float64
ANGLES = F  # float32: angles as an engine rounds them, which shows how much a model's logits hang on their last bits


def bf16_round(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).to(torch.bfloat16).to(t.dtype)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def causal_conv(u: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """u [T, C], weight [C, taps]: the newest input meets the last tap; nothing precedes the sequence."""
    n, taps = u.shape[0], weight.shape[1]
    out = torch.zeros_like(u)
    for t in range(n):
        for lag in range(min(taps, t + 1)):
            out[t] += weight[:, taps - 1 - lag] * u[t - lag]
    return out


def turn_halves(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, H, d]: element i < dims/2 of every head is paired with element i + dims/2; the rest pass."""
    half = dims // 2
    i = torch.arange(half, dtype=F)
    freq = base ** (-2.0 * i / max(dims, 1))
    a = (positions.to(ANGLES)[:, None] * freq.to(ANGLES)[None, :]).to(F)
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def visible_keys(n: int, size: Optional[int], keep_first: int = 0) -> torch.Tensor:
    """[queries, keys] of one sequence: the last `size` keys (own included) and the sequence's first `keep_first`."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    near = (i - j < size) if size is not None else torch.ones(n, n, dtype=torch.bool)
    return (j <= i) & (near | (j < keep_first))


def sink_softmax(scores: torch.Tensor, visible: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """scores [H, queries, keys], sink [H]: exp(s) / (exp(sink) + sum exp(s)) over the visible keys of each query."""
    s = scores.masked_fill(~visible[None], float("-inf"))
    m = torch.maximum(s.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (torch.exp(sink[:, None, None] - m) + e.sum(dim=-1, keepdim=True))


def turned(m: dict, x: torch.Tensor) -> torch.Tensor:
    rot = m.get("rot")
    if rot is None or not rot.get("dims"):
        return x
    return turn_halves(x, torch.arange(x.shape[0]), rot["dims"], rot["base"])


def latent_rows(w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, eps: float, rounded: bool = False) -> Tuple[torch.Tensor, torch.Tensor]:
    """What a layer with a W_dkv caches: the latent c [T, kv_rank] and the rotated key part [T, rot_dim]."""
    rd = bf16_round if rounded else (lambda t: t)
    down = rd(h @ w[p + "dkv"].T)
    rank = m["kv_rank"]
    c = rd(unit_rms(down[:, :rank], eps) * w[p + "dkv.norm"])
    return c, rd(turned(m, down[:, None, rank:])[:, 0])


def latent_attention(
    w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, c: torch.Tensor, key_part: torch.Tensor, rounded: bool = False,
) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    n, heads, dim, vdim = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rd(h @ w[p + "q"].T).reshape(n, heads, dim + m["rot_dim"])
    a, r = q[..., :dim], rd(turned(m, q[..., dim:]))
    k = rd(c @ w[p + "uk"].T).reshape(n, heads, dim)
    v = rd(c @ w[p + "uv"].T).reshape(n, heads, vdim)
    scores = torch.stack([(a[:, g] @ k[:, g].T + r[:, g] @ key_part.T) * m["scale"] for g in range(heads)])
    weights = sink_softmax(scores, visible_keys(n, (m.get("mask") or {}).get("size")), w[p + "sink"])
    out = torch.cat([weights[g] @ v[:, g] for g in range(heads)], dim=-1)
    return rd(out) @ w[p + "o"].T


def conv_projection(w: Dict[str, torch.Tensor], name: str, h: torch.Tensor, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    u = rd(h @ w[name].T + w[name + ".b"])
    return rd(causal_conv(u, w[name + ".conv"])) if name + ".conv" in w else u


def attention(w: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor, eps: float, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    n, heads, groups, dim = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = conv_projection(w, p + "q", h, rounded), conv_projection(w, p + "k", h, rounded)
    v = k.reshape(n, groups, dim)
    q = rd(turned(m, (unit_rms(q, eps) * w[p + "q.norm"]).reshape(n, heads, dim)))
    k = rd(turned(m, (unit_rms(k, eps) * w[p + "k.norm"]).reshape(n, groups, dim)))
    per = heads // groups
    scores = torch.stack([(q[:, g] @ k[:, g // per].T) * m["scale"] for g in range(heads)])
    mask = m.get("mask") or {}
    weights = sink_softmax(scores, visible_keys(n, mask.get("size"), mask.get("keep_first", 0)), torch.zeros(heads, dtype=h.dtype))
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = torch.cat([gate[:, g : g + 1] * (weights[g] @ v[:, g // per]) for g in range(heads)], dim=-1)
    return rd(out) @ w[p + "o"].T


def dense_ff(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    return rd(gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor, rounded: bool = False) -> torch.Tensor:
    rd = bf16_round if rounded else (lambda t: t)
    return rd(silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(logits: torch.Tensor, top: int, groups: Optional[dict] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """logits [T, E] -> (chosen [T, top], weights [T, top]): softmax over all; of the `groups.keep` groups of neighbours
    with the best members, the `top` largest scores."""
    s = torch.softmax(logits, dim=-1)
    allowed = s
    if groups is not None:
        members = s.reshape(s.shape[0], groups["count"], -1)
        kept = torch.topk(members.max(dim=-1).values, groups["keep"], dim=-1).indices
        open_ = torch.zeros(s.shape[0], groups["count"], dtype=torch.bool).scatter(1, kept, True)
        allowed = members.masked_fill(~open_[..., None], -1.0).reshape(s.shape)
    chosen = torch.topk(allowed, top, dim=-1).indices
    return chosen, torch.gather(s, 1, chosen)


def route_margin(logits: torch.Tensor, top: int, groups: Optional[dict] = None) -> torch.Tensor:
    """How far, as a share of the largest logit's size, the logits would have to move before another choice of groups or
    of experts came out (infinite where there is no other choice)."""
    size = logits.abs().max(dim=-1).values.clamp_min(1e-30)
    margin = torch.full(logits.shape[:-1], float("inf"), dtype=logits.dtype)
    allowed = logits
    if groups is not None:
        members = logits.reshape(logits.shape[0], groups["count"], -1)
        best = members.max(dim=-1).values
        if groups["keep"] < groups["count"]:
            ranked = torch.sort(best, dim=-1, descending=True).values
            margin = torch.minimum(margin, ranked[:, groups["keep"] - 1] - ranked[:, groups["keep"]])
        kept = torch.topk(best, groups["keep"], dim=-1).indices
        open_ = torch.zeros(best.shape, dtype=torch.bool).scatter(1, kept, True)
        allowed = members.masked_fill(~open_[..., None], float("-inf")).reshape(logits.shape)
    if top < logits.shape[-1]:
        ranked = torch.sort(allowed, dim=-1, descending=True).values
        margin = torch.minimum(margin, ranked[:, top - 1] - ranked[:, top])
    return margin / size


def expert_ff(w: Dict[str, torch.Tensor], p: str, mlp: dict, h: torch.Tensor, rounded: bool = False, margins: Optional[list] = None) -> torch.Tensor:
    logits = h @ w[p + "router"].T
    router = mlp["router"]
    if margins is not None:
        margins.append(route_margin(logits, router["top"], router.get("groups")))
    chosen, weights = route(logits, router["top"], router.get("groups"))
    out = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    for e in range(router["experts"]):
        share = (weights * (chosen == e)).sum(dim=-1)
        rows = torch.nonzero(share > 0)[:, 0]
        if rows.numel():
            out[rows] += share[rows, None] * expert(w, f"{p}e{e}.", h[rows], rounded)
    return out


def feed_forward(w: Dict[str, torch.Tensor], p: str, mlp: dict, h: torch.Tensor, rounded: bool = False, margins: Optional[list] = None) -> torch.Tensor:
    if mlp["kind"] == "dense":
        return dense_ff(w, p, h, rounded)
    if mlp["kind"] == "moe":
        return expert_ff(w, p, mlp, h, rounded, margins)
    raise ValueError(mlp["kind"])


def layer_kind(layer: dict) -> str:
    head, _, tail = layer["type"].rpartition("_")
    return head if tail.isdigit() else layer["type"]  # a numeric suffix marks another set of sizes of the same mixer


def forward(
    config: dict, w: Dict[str, torch.Tensor], tokens: List[int], rounded: bool = False, layers_out: Optional[list] = None,
    margins: Optional[list] = None,
) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  `rounded`: inputs of matrix products are rounded to bfloat16 where
    an engine that stores activations in bfloat16 would.  `layers_out` receives the residual after every layer,
    `margins` every router's margins [T] (see `route_margin`)."""
    rd = bf16_round if rounded else (lambda t: t)
    eps = config["norm"]["eps"]
    norm = lambda v, name: unit_rms(v, eps) * w[name]  # noqa: E731
    x = norm(w["embed"][torch.tensor(tokens, dtype=torch.long)], "embed.norm")
    latents: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = {}
    for i, layer in enumerate(config["layers"]):
        p, m, kind = f"l{i}.", layer["mixer"], layer_kind(layer)
        h = rd(norm(x, p + "norm1"))
        if kind == "latent_attention":
            if m.get("kv_from") is None:
                latents[i] = latent_rows(w, p + "mix.", m, h, eps, rounded)
            source = i if m.get("kv_from") is None else m["kv_from"]
            mixed = latent_attention(w, p + "mix.", m, h, *latents[source], rounded)
        elif kind == "attention":
            mixed = attention(w, p + "mix.", m, h, eps, rounded)
        else:
            raise ValueError(layer["type"])
        x = x + norm(mixed, p + "norm1b")
        if layer.get("mlp") is not None:
            x = x + norm(feed_forward(w, p + "mlp.", layer["mlp"], rd(norm(x, p + "norm2")), rounded, margins), p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    return rd(norm(x, "final.norm")) @ w["head"].T
