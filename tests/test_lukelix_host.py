"""Lukelix without a GPU: the configuration reader and its refusals, the tensors a model expects, the
cache each layer and the embedding ask for (pages read by several layers, state beside pages), and the plain
implementation's own rules against direct formulas."""

from __future__ import annotations

import json
import math

import pytest
import torch

import lukelix_tiny as lt
from plain import lukelix_plain as plain
from turboserve_amd.cache.layout import CacheLayout
from turboserve_amd.cache.storage import CacheStorage
from turboserve_amd.config.lukelix_config import LukelixConfig
from turboserve_amd.config.model_config import UnsupportedModelError
from turboserve_amd.config.registry import parse_model_config
from turboserve_amd.models.decoder import LayerCall
from turboserve_amd.parts.base import FixedState, PagedKV, PendingLayerNorm, ResidualStream, SharedKV
from turboserve_amd.parts.rope import banded_frequencies
from turboserve_amd.weights.random_init import describe_model


def test_the_reader_takes_every_size_from_the_file():
    config = parse_model_config(lt.CONFIG_A)
    assert isinstance(config, LukelixConfig)
    assert (config.vocab_size, config.hidden_size, config.norm_eps) == (211, 64, 1e-5)
    assert (config.bigram.buckets, config.bigram.mul_prev, config.bigram.mul_cur) == (97, 13, 5)
    assert [layer.type for layer in config.layers] == ["mamba2", "attention", "mamba2", "attention", "mamba2"]
    assert [layer.ff for layer in config.layers] == [40, None, None, 96, None]
    first, second, fourth = config.layers[0].mixer, config.layers[1].mixer, config.layers[3].mixer
    assert (first.heads, first.vdim, first.state, first.groups, first.taps, first.norm_groups) == (4, 16, 24, 2, 4, 2)
    assert (second.heads, second.kv_heads, second.dim, second.vdim, second.taps, second.scale) == (4, 2, 16, 24, 3, 0.3)
    assert (second.rot_base, second.rot_dims, second.kv_from) == (1000.0, 8, None)
    assert second.rot_scaling.as_mapping() == {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64.0}
    assert (fourth.kv_from, fourth.taps, fourth.scale) == (1, 2, 0.5)
    # What a file leaves out does not exist.
    other = parse_model_config(lt.CONFIG_B)
    assert other.layers[0].mixer.taps is None and other.layers[0].mixer.rot_scaling is None
    assert other.layers[3].mixer.rot_base is None and other.layers[3].mixer.kv_from is None
    assert parse_model_config(lt.CONFIG_C).bigram is None
    # Only layers with keys of their own take pages.
    assert config.kv_bytes_per_token(torch.bfloat16) == 2 * (16 + 24) * 2


@pytest.mark.parametrize("damage,message", [
    (lambda c: c["layers"][0].update(type="mamba"), "type"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=3), "norm_groups"),
    (lambda c: c["layers"][0]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), "factor"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("high"), "high"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=3), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=-1), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(dim=32), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(vdim=16), "kv_from"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda c: c["embedding"]["bigram"].update(mul_cur=-2), "mul_cur"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_the_reader_refuses(damage, message):
    config = json.loads(json.dumps(lt.CONFIG_A))
    damage(config)
    with pytest.raises(UnsupportedModelError, match=message):
        parse_model_config(config)


def test_a_layer_cannot_read_the_keys_of_a_layer_that_reads_others():
    config = json.loads(json.dumps(lt.CONFIG_B))
    config["layers"][5]["mixer"]["kv_from"] = 1
    with pytest.raises(UnsupportedModelError, match="kv_from"):
        parse_model_config(config)


def test_the_tensors_a_model_expects():
    _, model = describe_model(lt.CONFIG_A)
    specs = {name: spec.shape for name, spec in model.tensor_specs().items()}
    assert specs["embed"] == (211, 64) and specs["head"] == (211, 64) and specs["bigram"] == (98, 64)
    for norm in ("l0.norm1", "l0.norm2", "l1.norm1", "final.norm"):
        assert (specs[norm], specs[norm + ".b"]) == ((64,), (64,))
    assert "l1.norm2" not in specs and not any(name.startswith("l1.mlp") for name in specs)
    assert (specs["l0.mlp.up"], specs["l0.mlp.down"]) == ((40, 64), (64, 40))
    assert (specs["l1.mix.q"], specs["l1.mix.k"], specs["l1.mix.v"], specs["l1.mix.o"]) == ((64, 64), (32, 64), (48, 64), (64, 96))
    assert (specs["l1.mix.q.b"], specs["l1.mix.k.b"], specs["l1.mix.v.b"]) == ((64,), (32,), (48,)) and "l1.mix.o.b" not in specs
    assert (specs["l1.mix.q.conv"], specs["l1.mix.k.conv"], specs["l1.mix.v.conv"]) == ((64, 3), (32, 3), (48, 3))
    assert (specs["l1.mix.q.norm"], specs["l1.mix.k.norm"]) == ((16,), (16,))
    # A layer that reads another's keys has none of the key and value tensors.
    reader = {name.removeprefix("l3.mix."): shape for name, shape in specs.items() if name.startswith("l3.mix.")}
    assert reader == {"q": (64, 64), "q.b": (64,), "q.conv": (64, 2), "q.norm": (16,), "o": (64, 96)}
    # z | x | B | C | dt: 64 + 64 + 2 x 24 + 2 x 24 + 4 rows; the convolution runs over x, B and C.
    assert (specs["l0.mix.in"], specs["l0.mix.conv"], specs["l0.mix.conv.b"], specs["l0.mix.o"]) == ((228, 64), (160, 4), (160,), (64, 64))
    assert (specs["l0.mix.dt_bias"], specs["l0.mix.A_log"], specs["l0.mix.D"], specs["l0.mix.norm"]) == ((4,), (4,), (4,), (64,))
    assert "bigram" not in describe_model(lt.CONFIG_C)[1].tensor_specs()


def test_what_each_layer_and_the_embedding_ask_of_the_cache():
    _, model = describe_model(lt.CONFIG_A)
    needs = model.cache_needs()
    assert needs[0] == (FixedState((4, 16, 24)), FixedState((3, 64 + 48 + 48)))
    assert needs[1] == (PagedKV(2, 16, None, 24), FixedState((2, 64 + 32 + 48)))
    assert needs[3] == (SharedKV(2, 16, 24), FixedState((1, 64)))  # queries only: their projected rows are its own state
    assert needs[5] == FixedState((1,), torch.int32) and len(needs) == 6
    layout = CacheLayout.from_model(model)
    assert len(layout.groups) == 1 and layout.groups[0].entries == (1,)  # one set of pages for both attention layers
    assert layout.entry_units[1][0] == ("pages", 0, 0) and layout.entry_units[3][0] == ("shared", 0, 0)
    storage = CacheStorage(layout, [4], 8, 2, torch.float32, "cpu")
    views = storage.views()
    assert views[3][0].k.data_ptr() == views[1][0].k.data_ptr() and views[3][0].v.data_ptr() == views[1][0].v.data_ptr()
    assert views[1][0].writable and not views[3][0].writable and views[3][1].writable
    assert views[5].state.dtype == torch.int32 and views[5].state.shape == (3, 1)
    for state in storage.states:
        state.fill_(1)
    storage.zero_state_slots([1])
    assert all(float(state[1].abs().sum()) == 0 and bool((state[0] == 1).all()) and bool((state[2] == 1).all()) for state in storage.states)
    with pytest.raises(ValueError, match="state slots"):
        storage.zero_state_slots([3])
    # Without a convolution the reader keeps nothing of its own.
    _, other = describe_model(lt.CONFIG_C)
    assert other.cache_needs()[2] == (SharedKV(2, 32), FixedState((2, 192))) and other.cache_needs()[4] == PagedKV(1, 64)


def test_shared_pages_are_checked_against_what_their_owner_keeps():
    own = (PagedKV(2, 16, None, 24), FixedState((3,)))
    assert CacheLayout.from_needs([own, SharedKV(2, 16, 24)], [None, 0]).entry_units[1] == ("shared", 0, 0)
    with pytest.raises(ValueError, match="names none"):
        CacheLayout.from_needs([own, SharedKV(2, 16, 24)], [None, None])
    with pytest.raises(ValueError, match="reads 2 heads of 16/16"):
        CacheLayout.from_needs([own, SharedKV(2, 16)], [None, 0])
    with pytest.raises(ValueError, match="owns 0"):
        CacheLayout.from_needs([FixedState((3,)), SharedKV(2, 16)], [None, 0])
    windowed = PagedKV(2, 16, 20)
    with pytest.raises(ValueError, match="does not keep"):
        CacheLayout.from_needs([windowed, SharedKV(2, 16)], [None, 0])
    with pytest.raises(ValueError, match="does not keep"):
        CacheLayout.from_needs([windowed, SharedKV(2, 16, None, 21)], [None, 0])
    assert CacheLayout.from_needs([windowed, SharedKV(2, 16, None, 20)], [None, 0]).entry_units[1] == ("shared", 0, 0)
    # A call that reads another's cache and does not ask for shared pages reads all of it, as ever.
    assert CacheLayout.from_needs([own, None], [None, 0]).entry_units[1] == ("reads", 0)


def test_the_sizing_leaves_room_for_the_state():
    """Pages fill what the state tensors leave; a model of states alone is sized to no pages."""
    from turboserve_amd.cache.sizing import MemoryProfileError, size_cache
    from turboserve_amd.config.engine_config import SchedulerConfig

    scheduler = SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=32, block_size=8)
    state = FixedState((100, 5))
    pages = PagedKV(2, 8)
    layout = CacheLayout.from_needs([(pages, state), FixedState((1,), torch.int32)], [None, None])
    assert layout.state_bytes_per_slot() == 2004
    per_page = 2 * 16 * 8 * 2
    memory = (10 * per_page + 4 * 2004 + 5, 10 * per_page + 4 * 2004 + 5)
    sizing = size_cache(layout, scheduler, itemsize=2, gpu_memory_utilization=1.0, memory=memory)
    assert sizing.num_blocks == [10] and sizing.state_bytes == 4 * 2004
    alone = CacheLayout.from_needs([state], [None])
    assert size_cache(alone, scheduler, itemsize=2, gpu_memory_utilization=1.0, memory=memory).num_blocks == []
    with pytest.raises(MemoryProfileError):
        size_cache(alone, scheduler, itemsize=2, gpu_memory_utilization=1.0, memory=(2000, 2000))


def test_the_plan_names_the_calls_whose_keys_are_read():
    _, model = describe_model(lt.CONFIG_B)
    assert model.plan.schedule == tuple(LayerCall(i, cache_of=0 if i in (1, 5) else None) for i in range(6))
    assert [block.mixer.own_keys for block in model.blocks if hasattr(block.mixer, "own_keys")] == [True, False, True, False]


def test_a_pending_layer_norm_is_refused_by_norms_that_cannot_apply_it():
    from turboserve_amd.parts.base import PartSpec, Runtime
    from turboserve_amd.parts.registry import build_part

    runtime = Runtime(device=torch.device("cpu"), dtype=torch.float32, ops=None)
    rms = build_part("norm", PartSpec("rmsnorm", {"size": 4, "eps": 1e-6}), "n", runtime)
    layer = build_part("norm", PartSpec("layer_norm", {"size": 4, "eps": 1e-6}), "n", runtime)
    stream = ResidualStream(torch.zeros(1, 4), torch.zeros(1, 4), pending_norm=PendingLayerNorm(torch.ones(4), torch.zeros(4), 1e-6, 1.0))
    with pytest.raises(ValueError, match="layer norm"):
        rms.forward_residual(stream)
    layer.weight, layer.bias = torch.ones(4), torch.zeros(4)
    stream.pending_norm = (torch.ones(4), 1e-6, 1.0)
    with pytest.raises(ValueError, match="root-mean-square"):
        layer.forward_residual(stream)


# ---------------------------------------------------------------------------------------------
# the plain implementation's own rules
# ---------------------------------------------------------------------------------------------


def test_the_plain_bigram_rows():
    rule = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert plain.bigram_rows([4], rule) == [10]
    assert plain.bigram_rows([4, 5, 0, 9], rule) == [10, (12 + 35) % 10, 15 % 10, 63 % 10]


def test_the_plain_frequencies_keep_short_waves_and_stretch_long_ones():
    rot = {"base": 100.0, "dims": 12, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 40}}
    f, bare = plain.frequencies(rot), plain.frequencies({"base": 100.0, "dims": 12})
    kinds = []
    for stretched, own in zip(f, bare):
        wave = 2 * math.pi / own
        if wave < 40 / 4.0:
            assert stretched == own
            kinds.append("kept")
        elif wave > 40 / 1.0:
            assert stretched == pytest.approx(own / 8.0)
            kinds.append("divided")
        else:
            s = (40 / wave - 1.0) / 3.0
            assert stretched == pytest.approx((1 - s) * own / 8.0 + s * own) and own / 8.0 < stretched < own
            kinds.append("blended")
    assert set(kinds) == {"kept", "blended", "divided"}
    # The engine's tables hold the same frequencies.
    for base, dims, scaling in ((100.0, 12, rot["scaling"]), (500000.0, 64, {"factor": 4.0, "low": 2.0, "high": 3.0, "original": 512}),
                                (10.0, 8, {"factor": 3.0, "low": 0.5, "high": 9.0, "original": 20})):
        mine = banded_frequencies(dims, base, scaling)
        assert torch.allclose(mine, torch.tensor(plain.frequencies({"base": base, "dims": dims, "scaling": scaling}), dtype=torch.float64), rtol=1e-12)


def test_the_plain_rotation_turns_neighbouring_elements_of_the_first_only():
    rot = {"base": 100.0, "dims": 4}
    x = torch.randn(6, 2, 7, dtype=torch.float64)
    y = plain.turn_neighbours(x, rot)
    assert torch.equal(y[..., 4:], x[..., 4:]) and torch.allclose(y[0], x[0])
    for p in range(6):
        for i in range(2):
            a = p * 100.0 ** (-2 * i / 4)
            assert torch.allclose(y[p, :, 2 * i], x[p, :, 2 * i] * math.cos(a) - x[p, :, 2 * i + 1] * math.sin(a))
            assert torch.allclose(y[p, :, 2 * i + 1], x[p, :, 2 * i + 1] * math.cos(a) + x[p, :, 2 * i] * math.sin(a))


def test_the_plain_walk_is_a_weighted_sum_over_the_past():
    g = torch.Generator().manual_seed(1)
    T, N, P, rate, skip = 7, 3, 2, 0.7, 0.25
    x, B, C = (torch.randn(T, w, generator=g, dtype=torch.float64) for w in (P, N, N))
    dt = torch.rand(T, generator=g, dtype=torch.float64)
    y = plain.selective_walk(x, B, C, dt, rate, skip)
    for t in range(T):
        want = skip * x[t]
        for s in range(t + 1):
            want = want + math.exp(-rate * float(dt[s + 1:t + 1].sum())) * dt[s] * (C[t] @ B[s]) * x[s]
        assert torch.allclose(y[t], want)


def test_the_plain_gated_norm_takes_each_part_by_itself():
    y, z = torch.tensor([[1.0, 2.0, 30.0, 40.0]]), torch.full((1, 4), 50.0)  # silu(50) = 50
    out = plain.gated_group_norm(y, z, torch.tensor([1.0, 1.0, 1.0, 2.0]), 2, 0.0)
    assert torch.allclose(out, torch.tensor([[1 / 2.5 ** 0.5, 2 / 2.5 ** 0.5, 30 / 1250 ** 0.5, 2 * 40 / 1250 ** 0.5]]))


def test_the_plain_model_reads_another_layers_keys():
    """Changing the key matrix of the first layer moves what a later reader of its keys sees, also where the first
    layer's own output is switched off; the reader has no key tensors."""
    config = {"architecture": "Lukelix", "vocab": 30, "width": 16, "norm": {"eps": 1e-5}, "embedding": lt.bigram(7, 3, 2),
              "layers": [lt.layer(lt.attention(2, 1, 8, rot=8)), lt.layer(lt.attention(2, 1, 8, rot=8, kv_from=0))]}
    tensors = lt.draw_tensors(config, 1, torch.float64, 0.3)
    tensors["l0.mix.o"][:] = 0.0
    tokens = [3, 4, 5, 6, 7, 8]
    base = plain.forward(config, tensors, tokens)
    moved = dict(tensors, **{"l0.mix.k": tensors["l0.mix.k"] + 0.5 * torch.randn(8, 16, dtype=torch.float64)})
    assert float((plain.forward(config, moved, tokens)[-1] - base[-1]).abs().max()) > 1e-3
    # A sequence's first token takes the bigram table's last row.
    last = dict(tensors, bigram=tensors["bigram"].clone())
    last["bigram"][7] += 1.0
    assert float((plain.forward(config, last, tokens)[0] - base[0]).abs().max()) > 1e-3
