"""Ninenex without a GPU: the configuration reader and its refusals, the tensors a model expects, the
cache and state each layer asks for, layers that run with another's tensors, and the plain implementation's
own rules against direct formulas."""

from __future__ import annotations

import json
import math

import pytest
import torch

import ninenex_tiny as nt
from plain import ninenex_plain as plain
from turboserve_amd.cache.layout import CacheLayout
from turboserve_amd.config.model_config import UnsupportedModelError
from turboserve_amd.config.ninenex_config import DenseSizes, NinenexConfig, RoutedSizes
from turboserve_amd.config.registry import parse_model_config
from turboserve_amd.models.decoder import LayerCall
from turboserve_amd.parts.base import FixedState, PagedKV, PartSpec, Runtime
from turboserve_amd.parts.registry import build_part
from turboserve_amd.weights.random_init import describe_model


def test_the_reader_takes_every_size_from_the_file():
    config = parse_model_config(nt.CONFIG_A)
    assert isinstance(config, NinenexConfig)
    assert (config.vocab_size, config.hidden_size, config.norm_eps) == (211, 64, 1e-5)
    assert (config.embedding_scale, config.logit_scale) == (0.8, 2.0)
    assert [layer.type for layer in config.layers] == ["parallel", "mlstm", "mlstm", "mlstm", "parallel", "parallel", "mlstm"]
    assert [layer.weights_of for layer in config.layers] == [0, 1, 2, 1, 4, 0, 1]
    first, second, fifth = config.layers[0].mixer, config.layers[1].mixer, config.layers[4].mixer
    assert (first.left.heads, first.left.kv_heads, first.left.dim, first.left.vdim, first.left.scale) == (4, 2, 16, 24, 0.3)
    assert (first.left.chunk, first.left.rot_base, first.left.rot_dims) == (20, 1000.0, 8)
    assert (first.right.heads, first.right.dim, first.right.vdim, first.right.decay) == (2, 16, 24, (0.9, 0.99))
    assert (first.left_scale, first.right_scale, fifth.left_scale) == (0.7, 1.1, -0.4)
    assert (second.heads, second.dim, second.vdim, second.gate_cap) == (4, 16, 24, 9.0)
    assert config.layers[0].mlp == DenseSizes(48) and config.layers[2].mlp is None
    assert config.layers[1].mlp == RoutedSizes(40, 6, 2, 24) and config.layers[4].mlp == RoutedSizes(24, 4, 1, 0)
    # What a file leaves out does not exist.
    other = parse_model_config(nt.CONFIG_B)
    assert other.layers[2].mixer.left.chunk is None and other.layers[2].mixer.left.rot_base is None
    bare = {key: value for key, value in nt.CONFIG_B.items() if key not in ("embedding", "logit_scale")}
    assert (parse_model_config(bare).embedding_scale, parse_model_config(bare).logit_scale) == (1.0, 1.0)
    # Every layer that keeps keys has pages of its own, also one that runs with another's tensors.
    assert config.kv_bytes_per_token(torch.bfloat16) == (2 * 2 * (16 + 24) + (8 + 8)) * 2


@pytest.mark.parametrize("damage,message", [
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=3), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 1.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.0]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=0.5), "decay"),
    (lambda c: c["layers"][2]["mixer"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][2]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["layers"][4]["mlp"]["router"].update(top=5), "top"),
    (lambda c: c["layers"][1]["mlp"].update(shared={}), "shared"),
    (lambda c: c["layers"][3].update(weights_of=3), "weights_of"),
    (lambda c: c["layers"][3].update(weights_of=6), "weights_of"),
    (lambda c: c["layers"][3].update(weights_of=9), "weights_of"),
    (lambda c: c["layers"][3].update(weights_of=-1), "weights_of"),
    (lambda c: c["layers"][3].update(weights_of=2), "differs"),
    (lambda c: c["layers"][3]["mixer"].update(gate_cap=8.0), "differs"),
    (lambda c: c["embedding"].update(scale="large"), "scale"),
    (lambda c: c["norm"].update(eps=0), "eps"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_the_reader_refuses(damage, message):
    config = json.loads(json.dumps(nt.CONFIG_A))
    damage(config)
    with pytest.raises(UnsupportedModelError, match=message):
        parse_model_config(config)


def test_the_tensors_a_model_expects():
    _, model = describe_model(nt.CONFIG_A)
    specs = {name: spec.shape for name, spec in model.tensor_specs().items()}
    assert specs["embed"] == (211, 64) and specs["head"] == (211, 64)
    for norm in ("l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l2.norm1", "l2.norm1b", "final.norm"):
        assert specs[norm] == (64,) and norm + ".b" not in specs
    assert "l2.norm2" not in specs and not any(name.startswith("l2.mlp") for name in specs)
    # Layers that run with another's tensors have none.
    assert not any(name.startswith(("l3.", "l5.", "l6.")) for name in specs)
    left = {name.removeprefix("l0.mix.left."): shape for name, shape in specs.items() if name.startswith("l0.mix.left.")}
    assert left == {"q": (64, 64), "k": (32, 64), "v": (48, 64), "o": (64, 96), "q.b": (64,), "k.b": (32,), "v.b": (48,), "o.b": (64,)}
    right = {name.removeprefix("l0.mix.right."): shape for name, shape in specs.items() if name.startswith("l0.mix.right.")}
    assert right == {"q": (32, 64), "k": (32, 64), "v": (48, 64), "g": (48, 64), "o": (64, 48)}
    held = {name.removeprefix("l1.mix."): shape for name, shape in specs.items() if name.startswith("l1.mix.")}
    assert held == {"q": (64, 64), "k": (64, 64), "v": (96, 64), "g": (96, 64), "o": (64, 96), "norm": (96,), "i": (4, 64), "i.b": (4,),
                    "f": (4, 64), "f.b": (4,)}
    assert (specs["l0.mlp.gate"], specs["l0.mlp.gate.b"], specs["l0.mlp.up.b"], specs["l0.mlp.down.b"]) == ((48, 64), (48,), (48,), (64,))
    assert (specs["l1.mlp.router"], specs["l1.mlp.router.b"], specs["l1.mlp.e5.down"], specs["l1.mlp.shared.up"]) == ((6, 64), (6,), (64, 40), (24, 64))
    assert "l1.mlp.e0.gate.b" not in specs and "l1.mlp.shared.gate.b" not in specs and "l4.mlp.shared.gate" not in specs


def test_what_each_layer_asks_of_the_cache():
    _, model = describe_model(nt.CONFIG_A)
    needs = model.cache_needs()
    assert needs[0] == (PagedKV(2, 16, None, 24, 20), FixedState((2, 24, 16)))
    assert needs[1] == (FixedState((4, 24, 16)), FixedState((4, 16)), FixedState((4,)))
    assert needs[4] == (PagedKV(1, 8, None, None, 33), FixedState((3, 40, 8)))
    # A call with another layer's tensors asks for a cache or state of its own.
    assert model.plan.schedule == tuple(LayerCall(i) for i in (0, 1, 2, 1, 3, 0, 1)) and len(model.blocks) == 4
    assert needs[5] == needs[0] and needs[3] == needs[6] == needs[1]
    layout = CacheLayout.from_model(model)
    assert sorted((group.chunk, group.entries) for group in layout.groups) == [(20, (0, 5)), (33, (4,))]
    assert layout.state_bytes_per_slot() == 4 * (2 * 2 * 24 * 16 + 3 * 4 * (24 * 16 + 16 + 1) + 3 * (8 * 24 + 24 + 1) + 3 * 40 * 8)


def test_a_pair_runs_as_one_product_where_its_attention_can_place_its_heads():
    _, model = describe_model(nt.CONFIG_C)
    assert [block.mixer.fused for block in model.blocks if hasattr(block.mixer, "left")] == [True, False]


def test_the_parts_refuse_sizes_the_kernels_do_not_take():
    runtime = Runtime(device=torch.device("cpu"), dtype=torch.float32, ops=None)
    sizes = {"hidden_size": 8, "num_heads": 2, "head_dim": 4, "value_dim": 4, "norm_eps": 1e-6}
    with pytest.raises(ValueError, match="key channels"):
        build_part("mixer", PartSpec("mlstm", {**sizes, "head_dim": 513, "gate_cap": 3.0}), "m", runtime)
    with pytest.raises(ValueError, match="gate cap"):
        build_part("mixer", PartSpec("mlstm", {**sizes, "gate_cap": 0.0}), "m", runtime)
    with pytest.raises(ValueError, match="decay"):
        build_part("mixer", PartSpec("retention", {**sizes, "decay": (0.5, 1.01)}), "m", runtime)
    with pytest.raises(ValueError, match="positive"):
        build_part("mixer", PartSpec("retention", {**sizes, "value_dim": 0, "decay": (0.5, 1.0)}), "m", runtime)


# ---------------------------------------------------------------------------------------------
# the plain implementation's own rules
# ---------------------------------------------------------------------------------------------


def random(*shape, seed=1):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_the_plain_retention_is_a_weighted_sum_over_the_past():
    T, decay = 7, 0.8
    q, k, v = random(T, 3), random(T, 3, seed=2), random(T, 2, seed=3)
    out = plain.retention_walk(q, k, v, decay)
    for t in range(T):
        assert torch.allclose(out[t], sum(decay ** (t - s) * (q[t] @ k[s]) * v[s] for s in range(t + 1)))


def test_the_plain_memory_is_the_unscaled_one_where_nothing_is_clipped():
    """The running maximum only rescales state and sum: o = (sum_s w_s (q . k_s) v_s) / (max(|sum_s w_s q . k_s|, 1) + 1e-6 exp(m)),
    w_s = exp(f_(s+1) + .. + f_t + i_s)."""
    T = 9
    q, k, v = random(T, 3), random(T, 3, seed=2), random(T, 2, seed=3)
    i, f = 2.0 * random(T, seed=4), -random(T, seed=5).abs()
    out = plain.memory_walk(q, k, v, i, f)
    m = 0.0
    for t in range(T):
        weights = [math.exp(float(f[s + 1:t + 1].sum() + i[s])) for s in range(t + 1)]
        m = max(float(f[t]) + m, float(i[t]))
        top = sum(w * (q[t] @ k[s]) * v[s] for s, w in enumerate(weights))
        low = max(abs(float(sum(w * (q[t] @ k[s]) for s, w in enumerate(weights)))), 1.0) + 1e-6 * math.exp(m)
        assert torch.allclose(out[t], top / low)


def test_the_plain_gates_are_capped():
    i, f = plain.capped_gates(torch.tensor([100.0, -100.0, 0.1]), torch.tensor([100.0, -100.0, 0.0]), 5.0)
    assert torch.allclose(i, torch.tensor([5.0, -5.0, 5.0 * math.tanh(0.02)]))
    assert torch.allclose(f, torch.tensor([-math.log1p(math.exp(-5.0)), -5.0 - math.log1p(math.exp(-5.0)), -math.log(2.0)]))


def test_the_plain_chunks_and_rotation():
    assert [plain.sees(7, j, 3) for j in range(9)] == [False] * 6 + [True, True, False]
    assert plain.sees(7, 0, None) and not plain.sees(7, 8, None) and plain.sees(4, 4, 1) and not plain.sees(4, 3, 1)
    rot, x = {"base": 100.0, "dims": 4}, random(6, 2, 7)
    y = plain.turn_halves(x, rot)
    assert torch.equal(y[..., 4:], x[..., 4:]) and torch.allclose(y[0], x[0])
    for p in range(6):
        for i in range(2):
            a = p * 100.0 ** (-2 * i / 4)
            assert torch.allclose(y[p, :, i], x[p, :, i] * math.cos(a) - x[p, :, i + 2] * math.sin(a))
            assert torch.allclose(y[p, :, i + 2], x[p, :, i + 2] * math.cos(a) + x[p, :, i] * math.sin(a))


def test_the_plain_router_weighs_the_chosen_logits_only():
    z = torch.tensor([0.5, 2.0, -1.0, 1.0])
    (a, wa), (b, wb) = plain.chosen(z, 2)
    assert (a, b) == (1, 3) and float(wa) == pytest.approx(math.exp(2.0) / (math.exp(2.0) + math.exp(1.0))) and float(wa + wb) == pytest.approx(1.0)


def test_the_plain_model_runs_a_layer_with_anothers_tensors():
    layers = [nt.layer(nt.memory(2, 4, 4, 3.0), nt.dense(8))]
    config = nt.model([*layers, nt.again(layers, 0)], vocab=20, width=8)
    tensors = nt.draw_tensors(config, 1, torch.float64, 0.3)
    assert not any(name.startswith("l1.") for name in tensors)
    copied = nt.model([layers[0], layers[0]], vocab=20, width=8)
    both = {**tensors, **{"l1." + name[3:]: t for name, t in tensors.items() if name.startswith("l0.")}}
    tokens = [3, 4, 5, 6]
    assert torch.equal(plain.forward(config, tensors, tokens), plain.forward(copied, both, tokens))
