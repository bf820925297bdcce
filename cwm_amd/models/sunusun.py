"""The Sunusun decoder as a plan of parts.

An embedding with sinusoidal positions; pre-norm layers whose norms have one number for all coordinates; the mixer is an
attention (a norm of every query and key head, queries that grow with their position, scores that fall with the distance,
one added to the softmax's denominator) side by side with a gated recurrence, each result normalised over the width and
half of their sum taken, or an RWKV time mixing; the feed-forward is dense with the erf form of gelu.  A layer may use
another layer's tensors with a cache or state of its own: the run order then names that layer again.  The factor on the
logits rides on the final norm.
Tensor names: `embed`, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.left.{q,k,v,q.norm,k.norm,r1,r2,o,out}` with
`l<i>.mix.right.{z,z.b,x,x.b,g,o,out}`, or `l<i>.mix.{mu.{r,k,v,g,w},r,k,v,g,w1,w2,w0,u,norm,o}`, `l<i>.mlp.{up,down}`,
`final.norm`, `head`.
"""

from __future__ import annotations

from typing import Dict

from ..config.registry import register_architecture
from ..config.sunusun import ParallelConfig, SunusunConfig, WKVConfig
from ..parts.base import LayerCall, LayerPlan, ModelPlan, PartChoice, PartSlot

ARCHITECTURE_NAME = "Sunusun"
POSITION_BASE = 10000.0  # of the sinusoidal positions: the design fixes it
SIDE_SHARE = 0.5  # of each of the two results side by side


def _parallel(width: int, eps: float, sizes: ParallelConfig) -> PartChoice:
    left = sizes.left
    attention = PartChoice(
        "head_norm_attention",
        {
            "dim": width, "n_heads": left.heads, "n_kv_heads": left.kv_heads, "qk_dim": left.dim, "v_dim": left.vdim, "scale": left.scale,
            "bias": False, "qk_norm": True, "eps": eps, "gate": False, "distance_bias": True, "unit_sink": True,
            "query_temperature": (left.q_temp.coef, left.q_temp.every) if left.q_temp is not None else None,
        },
    )
    recurrence = PartChoice("min_gru", {"dim": width, "width": sizes.right.width})
    return PartChoice("side_by_side", {"mixers": {"left": (attention, SIDE_SHARE), "right": (recurrence, SIDE_SHARE)}, "out_norm": eps, "dim": width})


def build_plan(config: SunusunConfig) -> ModelPlan:
    width, eps = config.width, config.norm.eps
    norm = {"dim": width, "eps": eps, "tensor": "", "scalar": True}
    layers, plan_of = [], {}  # type: ignore[var-annotated]
    for i, layer in enumerate(config.layers):
        if config.owner(i) != i:
            continue
        sizes = layer.mixer_config()
        if isinstance(sizes, ParallelConfig):
            mixer = _parallel(width, eps, sizes)
        elif isinstance(sizes, WKVConfig):
            mixer = PartChoice("wkv", {"dim": width, "heads": sizes.heads, "head_dim": sizes.dim, "eps": eps})
        else:  # pragma: no cover  (LayerConfig has refused it)
            raise TypeError(f"layer {i}: no part for {type(sizes).__name__}")
        parts: Dict[str, PartSlot] = {
            "norm1": PartSlot("norm", PartChoice("rmsnorm", norm), "norm1"),
            "mixer": PartSlot("mixer", mixer, "mix."),
            "norm2": PartSlot("norm", PartChoice("rmsnorm", {**norm, "optional": layer.mlp is None}), "norm2"),
        }
        if layer.mlp is not None:
            parts["feed_forward"] = PartSlot(
                "feed_forward", PartChoice("activated_mlp", {"dim": width, "hidden_dim": layer.mlp.ff, "activation": "gelu_erf"}), "mlp.",
            )
        plan_of[i] = len(layers)
        layers.append(LayerPlan(prefix=f"l{i}.", block="pre_norm", parts=parts))
    sizes = {"vocab_size": config.vocab, "dim": width, "tensor": ""}
    return ModelPlan(
        vocab_size=config.vocab,
        dim=width,
        layers=layers,
        run_order=[LayerCall(layer=plan_of[config.owner(i)]) for i in range(len(config.layers))],
        embedding=PartSlot("embedding", PartChoice("sinusoidal_embedding", {**sizes, "base": POSITION_BASE}), "embed"),
        final_norm=PartSlot("norm", PartChoice("rmsnorm", {**norm, "gain": config.logit_scale}), "final.norm"),
        head=PartSlot("head", PartChoice("linear_head", sizes), "head"),
        max_positions=config.max_positions,
    )


register_architecture(ARCHITECTURE_NAME, SunusunConfig, build_plan)
