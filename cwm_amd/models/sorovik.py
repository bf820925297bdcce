"""The Sorovik decoder as a plan of parts.

A normed embedding; layers whose sublayers read a norm of the residual and pass another before they join it.  The mixer is
an attention through a cached latent (a sliding window, a sink, rotation in halves of a shared key part; a layer may read
an earlier layer's cached rows instead of making its own) or an attention whose queries and keys pass a short convolution
and a norm over the whole projection, whose values are the keys, with kept first tokens beside its window, one added to
the softmax's denominator and a gate a head.  The feed-forward is dense and gated (the tanh form of gelu) or routed experts chosen from
the best groups.  Tensor names: `embed`, `embed.norm`, `l<i>.norm1`, `l<i>.norm1b`, `l<i>.norm2`, `l<i>.norm2b`,
`l<i>.mix.{q,dkv,dkv.norm,uk,uv,sink,o}` or `l<i>.mix.{q,q.b,q.conv,q.norm,k,k.b,k.conv,k.norm,g,o}`,
`l<i>.mlp.{gate,up,down}` or `l<i>.mlp.{router,e<j>.gate,e<j>.up,e<j>.down}`, `final.norm`, `head`.
"""

from __future__ import annotations

from typing import Dict, Optional

from ..config.registry import register_architecture
from ..config.sorovik import AttentionConfig, FeedForwardConfig, LatentAttentionConfig, RotationConfig, SorovikConfig
from ..parts.base import LayerCall, LayerPlan, ModelPlan, PartChoice, PartSlot

ARCHITECTURE_NAME = "Sorovik"


def _rotation(rot: Optional[RotationConfig]) -> Optional[PartChoice]:
    if rot is None or rot.dims == 0:
        return None
    return PartChoice("rotary", {"head_dim": rot.dims, "theta": rot.base, "pairing": "halves"})


def _latent(width: int, eps: float, sizes: LatentAttentionConfig, cache_window: Optional[int]) -> PartChoice:
    return PartChoice(
        "latent_attention",
        {
            "dim": width, "n_heads": sizes.heads, "head_dim": sizes.dim, "rot_dim": sizes.rot_dim, "v_dim": sizes.vdim, "kv_rank": sizes.kv_rank,
            "q_rank": None, "scale": sizes.scale, "eps": eps, "window": sizes.mask.size if sizes.mask is not None else None,
            "cache_window": cache_window, "sink": True, "gate": False, "own_kv": sizes.kv_from is None, "position_encoding": _rotation(sizes.rot),
        },
    )


def _attention(width: int, eps: float, sizes: AttentionConfig) -> PartChoice:
    return PartChoice(
        "conv_attention",
        {
            "dim": width, "n_heads": sizes.heads, "n_kv_heads": sizes.kv_heads, "head_dim": sizes.dim, "scale": sizes.scale,
            "window": sizes.mask.size if sizes.mask is not None else None, "keep_first": sizes.mask.keep_first if sizes.mask is not None else 0,
            "taps": sizes.conv, "bias": True, "qk_norm": True, "eps": eps, "unit_sink": True, "gate": True, "position_encoding": _rotation(sizes.rot),
        },
    )


def _feed_forward(width: int, mlp: FeedForwardConfig) -> PartChoice:
    if mlp.kind == "dense":
        return PartChoice("gated_mlp", {"dim": width, "hidden_dim": mlp.ff, "activation": "gelu_tanh"})
    groups = mlp.router.groups
    return PartChoice(
        "routed_experts",
        {
            "dim": width, "hidden_dim": mlp.expert.ff, "n_experts": mlp.router.experts, "top": mlp.router.top, "scores": "softmax_all",
            "groups": (groups.count, groups.keep) if groups is not None else None, "activation": "silu",
        },
    )


def cache_windows(config: SorovikConfig) -> Dict[int, Optional[int]]:
    """For every layer with a latent of its own: the longest window through which it or a layer that reads its rows looks
    back (None: all keys), which is what its cache keeps."""
    spans: Dict[int, Optional[int]] = {}
    for i, layer in enumerate(config.layers):
        m = layer.mixer_config()
        if not isinstance(m, LatentAttentionConfig):
            continue
        owner = i if m.kv_from is None else m.kv_from
        size = m.mask.size if m.mask is not None else None
        if owner not in spans:
            spans[owner] = size
        elif spans[owner] is not None:
            spans[owner] = None if size is None else max(spans[owner], size)
    return spans


def build_plan(config: SorovikConfig) -> ModelPlan:
    width, eps = config.width, config.norm.eps
    norm = PartChoice("rmsnorm", {"dim": width, "eps": eps, "tensor": ""})
    unread = PartChoice("rmsnorm", {"dim": width, "eps": eps, "tensor": "", "optional": True})
    spans = cache_windows(config)
    layers, order = [], []
    for i, layer in enumerate(config.layers):
        sizes = layer.mixer_config()
        call = LayerCall(layer=i)
        if isinstance(sizes, LatentAttentionConfig):
            mixer = _latent(width, eps, sizes, spans[i if sizes.kv_from is None else sizes.kv_from])
            if sizes.kv_from is not None:
                call = LayerCall(layer=i, cache_of=sizes.kv_from)
        elif isinstance(sizes, AttentionConfig):
            mixer = _attention(width, eps, sizes)
        else:  # pragma: no cover  (LayerConfig has refused it)
            raise TypeError(f"layer {i}: no part for {type(sizes).__name__}")
        parts = {
            "norm1": PartSlot("norm", norm, "norm1"),
            "mixer": PartSlot("mixer", mixer, "mix."),
            "norm1b": PartSlot("norm", norm, "norm1b"),
        }
        if layer.mlp is not None:
            parts["norm2"] = PartSlot("norm", norm, "norm2")
            parts["feed_forward"] = PartSlot("feed_forward", _feed_forward(width, layer.mlp), "mlp.")
            parts["norm2b"] = PartSlot("norm", norm, "norm2b")
        else:  # a folder may hold the norms of a sublayer that the layer does not have
            parts["norm2"] = PartSlot("norm", unread, "norm2")
            parts["norm2b"] = PartSlot("norm", unread, "norm2b")
        layers.append(LayerPlan(prefix=f"l{i}.", block="sandwich_norm", parts=parts))
        order.append(call)
    sizes = {"vocab_size": config.vocab, "dim": width, "tensor": ""}
    embedding_norm = PartChoice("group_rmsnorm", {"dim": width, "eps": eps, "groups": 1, "tensor": ""})
    return ModelPlan(
        vocab_size=config.vocab,
        dim=width,
        layers=layers,
        run_order=order,
        embedding=PartSlot("embedding", PartChoice("normed_embedding", {**sizes, "norm": embedding_norm, "norm_prefix": ".norm"}), "embed"),
        final_norm=PartSlot("norm", norm, "final.norm"),
        head=PartSlot("head", PartChoice("linear_head", sizes), "head"),
        max_positions=config.max_positions,
    )


register_architecture(ARCHITECTURE_NAME, SorovikConfig, build_plan)
