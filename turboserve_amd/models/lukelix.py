"""Lukelix: from its configuration to a plan of parts.

A decoder whose parts read the stream itself and whose norms stand behind them, ``x += norm1(mix(x))``, ``x +=
norm2(ff(x))``, every norm a layer norm with weight and bias.  The stream starts as the token's row of ``embed`` plus a
row of ``bigram`` hashed from the token and the one before it; behind ``final.norm`` the output matrix ``head`` makes
the logits.  Each layer is described on its own, with one of two mixers:

* ``attention``: causal grouped-query attention with biased projections, a short convolution over time on q, k and v, a
  norm per q and k head with one gain for all heads, rotation of neighbouring pairs over a head's first elements with
  stretched long wavelengths; a layer with ``kv_from`` has queries only and reads that layer's cached keys and values.
* ``mamba2``: a selective state space (a short convolution with bias and silu over x, B and C, a decay per head and
  token, a 32-bit state per head, a gated norm in equal parts).

Feed-forward: ``down(max(up(x), 0)^2)``, or none.  Tensors are named ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.mix.q.conv``,
``l<i>.mlp.up`` and so on, without a ``weight`` suffix; a bias is ``<tensor>.b``.
"""

from __future__ import annotations

from turboserve_amd.config.lukelix_config import AttentionSizes, LukelixConfig, Mamba2Sizes
from turboserve_amd.models.decoder import LayerCall, LayerSpec, ModelPlan
from turboserve_amd.parts.base import PartSpec

#: Positions the rotary tables are first made for; they grow by doubling.
INITIAL_POSITIONS = 4096

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}


def _attention(width: int, eps: float, sizes: AttentionSizes) -> PartSpec:
    position = PartSpec("none", {})
    if sizes.rot_base is not None:
        position = PartSpec("rope", {
            "head_dim": sizes.rot_dims, "theta": sizes.rot_base, "max_positions": INITIAL_POSITIONS, "exact": True, "neighbours": True,
            "bands": None if sizes.rot_scaling is None else sizes.rot_scaling.as_mapping(),
        })
    return PartSpec("gqa_attention", {
        "hidden_size": width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
        "value_dim": sizes.vdim, "scale": sizes.scale, "qkv_bias": True, "out_bias": False, "window": None, "position": position,
        "head_norm": {"eps": eps, "gain_offset": 0.0}, "conv": None if sizes.taps is None else {"taps": sizes.taps, "suffix": "conv"},
        "own_keys": sizes.kv_from is None, "names": ATTENTION_NAMES,
    })


def _mamba2(width: int, eps: float, sizes: Mamba2Sizes) -> PartSpec:
    return PartSpec("mamba2", {
        "hidden_size": width, "num_heads": sizes.heads, "value_dim": sizes.vdim, "state_dim": sizes.state, "groups": sizes.groups,
        "taps": sizes.taps, "norm_groups": sizes.norm_groups, "norm_eps": eps,
    })


def lukelix_plan(config: LukelixConfig) -> ModelPlan:
    width = config.hidden_size
    norm = PartSpec("layer_norm", {"size": width, "eps": config.norm_eps, "weight_name": ""})
    layers, schedule = [], []
    for index, layer in enumerate(config.layers):
        mixer = (_attention if isinstance(layer.mixer, AttentionSizes) else _mamba2)(width, config.norm_eps, layer.mixer)
        feed_forward = None
        if layer.ff is not None:
            feed_forward = PartSpec("mlp", {"hidden_size": width, "intermediate_size": layer.ff, "activation": "relu_squared",
                                            "names": ("up", "down")})
        block = PartSpec("sandwich", {
            "mixer": mixer, "feed_forward": feed_forward, "norm": norm, "pre_norm": PartSpec("plain_sum", {"size": width}),
            "mixer_name": "mix", "ff_name": "mlp", "mixer_post_name": "norm1", "ff_post_name": "norm2",
        })
        layers.append(LayerSpec(prefix=f"l{index}", block=block))
        schedule.append(LayerCall(index, cache_of=getattr(layer.mixer, "kv_from", None)))
    table = {"vocab_size": config.vocab_size, "hidden_size": width, "weight_name": ""}
    embedding = PartSpec("token_table", table)
    if config.bigram is not None:
        embedding = PartSpec("token_table_bigram", {**table, "buckets": config.bigram.buckets, "mul_prev": config.bigram.mul_prev,
                                                    "mul_cur": config.bigram.mul_cur, "pairs_name": "bigram"})
    return ModelPlan(
        vocab_size=config.vocab_size,
        hidden_size=width,
        layers=tuple(layers),
        schedule=tuple(schedule),
        embedding=embedding,
        head=PartSpec("norm_linear", {"vocab_size": config.vocab_size, "hidden_size": width, "norm": norm,
                                      "norm_prefix": "final.norm", "tied_to": None, "weight_name": ""}),
        embedding_prefix="embed",
        head_prefix="head",
    )
