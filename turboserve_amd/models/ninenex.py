"""Ninenex: from its configuration to a plan of parts.

A decoder with a norm before and behind each part, ``x += norm1b(mix(norm1(x)))``, ``x += norm2b(ff(norm2(x)))``, every norm
a layer norm with a weight and no bias.  The stream starts as the token's row of ``embed`` times a constant; behind
``final.norm`` the output matrix ``head`` makes the logits, which leave times another.  Each layer is described on its own,
with one of two mixers:

* ``mlstm``: the matrix memory of xLSTM (exponential gates with a capped logarithm, a running maximum, a sum of keys that
  normalises the read-out).
* ``parallel``: two mixers that read the same input, their outputs added with a weight each.  ``left`` is grouped-query
  attention with biased projections, rotation in halves of a head's first elements and chunks of positions; ``right`` is
  retention.

Feed-forward: a dense gated one with biases and the tanh form of GELU on the gate, a routed one (a biased router whose
weights are the softmax over the taken experts, silu experts, a shared expert), or none.  A layer may run with another
layer's tensors; its cache or state is its own.  Tensors are named ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.mix.left.q``,
``l<i>.mlp.e<j>.gate`` and so on, without a ``weight`` suffix; a bias is ``<tensor>.b``.
"""

from __future__ import annotations

from turboserve_amd.config.ninenex_config import (
    ChunkedAttentionSizes,
    DenseSizes,
    MatrixMemorySizes,
    NinenexConfig,
    ParallelSizes,
    RetentionSizes,
    RoutedSizes,
)
from turboserve_amd.kernels.ops import GELU_TANH_RULE
from turboserve_amd.models.decoder import LayerCall, LayerSpec, ModelPlan
from turboserve_amd.parts.base import PartSpec

#: Positions the rotary tables are first made for; they grow by doubling.
INITIAL_POSITIONS = 4096

GLU_NAMES = ("gate", "up", "down")
ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o"}


def _chunked_attention(width: int, sizes: ChunkedAttentionSizes) -> PartSpec:
    position = PartSpec("none", {})
    if sizes.rot_base is not None:
        position = PartSpec("rope", {"head_dim": sizes.rot_dims, "theta": sizes.rot_base, "max_positions": INITIAL_POSITIONS, "exact": True})
    return PartSpec("gqa_attention", {
        "hidden_size": width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
        "value_dim": sizes.vdim, "scale": sizes.scale, "qkv_bias": True, "out_bias": True, "window": None, "position": position,
        "chunk": sizes.chunk, "names": ATTENTION_NAMES,
    })


def _retention(width: int, eps: float, sizes: RetentionSizes) -> PartSpec:
    return PartSpec("retention", {"hidden_size": width, "num_heads": sizes.heads, "head_dim": sizes.dim, "value_dim": sizes.vdim,
                                  "decay": sizes.decay, "norm_eps": eps})


def _mixer(width: int, eps: float, sizes) -> PartSpec:
    if isinstance(sizes, MatrixMemorySizes):
        return PartSpec("mlstm", {"hidden_size": width, "num_heads": sizes.heads, "head_dim": sizes.dim, "value_dim": sizes.vdim,
                                  "gate_cap": sizes.gate_cap, "norm_eps": eps})
    if isinstance(sizes, ParallelSizes):
        return PartSpec("mixer_pair", {
            "left": _chunked_attention(width, sizes.left), "right": _retention(width, eps, sizes.right),
            "left_scale": sizes.left_scale, "right_scale": sizes.right_scale,
        })
    raise TypeError(f"no mixer for {sizes!r}")


def _feed_forward(width: int, sizes) -> PartSpec | None:
    if sizes is None:
        return None
    if isinstance(sizes, DenseSizes):
        return PartSpec("swiglu", {"hidden_size": width, "intermediate_size": sizes.ff, "names": GLU_NAMES, "rule": GELU_TANH_RULE,
                                   "bias": True})
    if isinstance(sizes, RoutedSizes):
        shared = None
        if sizes.shared_ff:
            shared = PartSpec("swiglu", {"hidden_size": width, "intermediate_size": sizes.shared_ff, "names": GLU_NAMES})
        return PartSpec("routed_experts", {
            "hidden_size": width, "expert_size": sizes.ff, "experts": sizes.experts, "top": sizes.top, "router_scores": "softmax",
            "router_bias_name": "router.b", "shared": shared,
        })
    raise TypeError(f"no feed-forward for {sizes!r}")


def ninenex_plan(config: NinenexConfig) -> ModelPlan:
    width = config.hidden_size
    norm = PartSpec("layer_norm", {"size": width, "eps": config.norm_eps, "weight_name": "", "bias_name": None})
    layers, place = [], {}
    for index, layer in enumerate(config.layers):
        if layer.weights_of != index:
            continue
        place[index] = len(layers)
        layers.append(LayerSpec(prefix=f"l{index}", block=PartSpec("sandwich", {
            "mixer": _mixer(width, config.norm_eps, layer.mixer), "feed_forward": _feed_forward(width, layer.mlp), "norm": norm,
        })))
    return ModelPlan(
        vocab_size=config.vocab_size,
        hidden_size=width,
        layers=tuple(layers),
        schedule=tuple(LayerCall(place[layer.weights_of]) for layer in config.layers),
        embedding=PartSpec("token_table", {"vocab_size": config.vocab_size, "hidden_size": width, "weight_name": "",
                                           "scale": config.embedding_scale}),
        head=PartSpec("norm_linear", {"vocab_size": config.vocab_size, "hidden_size": width, "norm": norm, "norm_prefix": "final.norm",
                                      "tied_to": None, "weight_name": "", "scale": config.logit_scale}),
        embedding_prefix="embed",
        head_prefix="head",
    )
