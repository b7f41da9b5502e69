"""Small Ninenex configurations that differ in every size, constant and layer order, and helpers that
write their random model folders and compute the plain implementation's logits."""

from __future__ import annotations

import json
from pathlib import Path

import torch

from plain import ninenex_plain as plain


def memory(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def attention(heads, kv_heads, dim, vdim=None, chunk=None, scale=None, rot=None, base=10000.0):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim if vdim is None else vdim,
            "scale": dim ** -0.5 if scale is None else scale}
    if chunk is not None:
        left["mask"] = {"size": chunk}
    if rot is not None:
        left["rot"] = {"base": base, "dims": rot}
    return left


def retention(heads, dim, vdim, *decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def parallel(left, right, left_scale, right_scale):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            "shared": None if shared is None else {"ff": shared}}


def layer(mixer, mlp=None):
    return {**mixer, "mlp": mlp}


def again(layers: list[dict], index: int) -> dict:
    """The entry of a layer that runs with layer ``index``'s tensors."""
    return {**layers[index], "weights_of": index}


def model(layers, *, vocab=61, width=40, eps=1e-5, embedding=1.5, logits=0.7):
    return {"architecture": "Ninenex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embedding},
            "logit_scale": logits, "layers": layers}


#: A: a chunk of no multiple of the page; values wider than keys; a memory without a feed-forward; three layers that run with
#: another's tensors, one of them with those of a layer that itself does; experts with and without a shared one.
_A = [
    layer(parallel(attention(4, 2, 16, 24, chunk=20, scale=0.3, rot=8, base=1000.0), retention(2, 16, 24, 0.9, 0.99), 0.7, 1.1), dense(48)),
    layer(memory(4, 16, 24, 9.0), moe(6, 2, 40, 24)),
    layer(memory(3, 24, 8, 15.0)),
]
_A.append(again(_A, 1))
_A.append(layer(parallel(attention(6, 1, 8, chunk=33, rot=8), retention(3, 8, 40, 0.5, 0.999, 1.0), -0.4, 0.6), moe(4, 1, 24)))
_A.append(again(_A, 0))
_A.append({**_A[3], "weights_of": 3})
CONFIG_A = model(_A, vocab=211, width=64, embedding=0.8, logits=2.0)
PAGE_A = 16

#: B: sizes that 16-byte accesses do not divide; one head; as many key heads as query heads; a chunk of one token and one
#: shorter than a page; no chunk and no rotation; every expert taken; constants of 1; a state row alone.
CONFIG_B = model([
    layer(memory(1, 20, 7, 4.0), dense(28)),
    layer(parallel(attention(3, 3, 12, 20, chunk=7, scale=0.5, rot=2, base=50.0), retention(1, 9, 6, 0.8), 1.0, 1.0), moe(3, 3, 20, 12)),
    layer(parallel(attention(1, 1, 20), retention(5, 4, 11, 0.1, 0.7, 0.9, 0.97, 1.0), 0.3, 1.4)),
    layer(memory(5, 1, 33, 20.0), moe(5, 4, 12)),
    layer(parallel(attention(4, 2, 12, 8, chunk=1), retention(2, 33, 12, 0.95, 0.6), 0.9, 0.2), dense(20)),
], vocab=97, width=51, eps=1e-6, embedding=1.0, logits=1.0)
PAGE_B = 8

#: C: sizes of the matrix-core kernels: long portions cut into pieces in every state layer, attention of whole heads
#: turned with a chunk of two pages, plain causal attention (which is not placed beside the retention), pages of 32.
CONFIG_C = model([
    layer(parallel(attention(6, 2, 32, chunk=64, scale=0.25, rot=32, base=200000.0), retention(4, 32, 64, 0.99, 0.95, 0.999, 0.8), 0.6, 0.8), dense(96)),
    layer(memory(2, 64, 72, 12.0), moe(8, 3, 32, 40)),
    layer(parallel(attention(4, 1, 64, rot=16), retention(2, 136, 8, 0.9, 0.998), 0.8, 0.5)),
    layer(memory(1, 136, 32, 8.0), dense(64)),
], vocab=160, width=96, eps=1e-6, embedding=3.0, logits=0.25)
PAGE_C = 32

TINY = {"A": (CONFIG_A, 41, PAGE_A), "B": (CONFIG_B, 42, PAGE_B), "C": (CONFIG_C, 43, PAGE_C)}


def draw_tensors(config: dict, seed: int, dtype: torch.dtype, std: float) -> dict[str, torch.Tensor]:
    """Random tensors by the names and shapes the engine's own description of the model gives (the plain
    implementation reads them by name): matrices N(0, std); gains around one; biases, routers and gates wide enough to
    matter (forget gates from a few tokens to hundreds)."""
    from turboserve_amd.weights.random_init import describe_model

    _, described = describe_model(config)
    generator = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, spec in described.tensor_specs().items():
        values = torch.randn(spec.shape, generator=generator)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
            values = 1.0 + 0.3 * values
        elif name == "embed":
            values = 0.7 * values
        elif name.endswith(".f.b"):
            values = 2.5 + 1.5 * values
        elif leaf == "b":
            values = 0.4 * values
        elif leaf == "router":
            values = 4.0 * std * values
        elif leaf in ("i", "f"):
            values = 2.0 * std * values
        else:
            values = std * values
        tensors[name] = values.to(dtype).contiguous()
    return tensors


def make_model_dir(folder: Path, config: dict, seed: int, dtype: torch.dtype = torch.float32, std: float = 0.15,
                   tensors: dict[str, torch.Tensor] | None = None) -> Path:
    from safetensors.torch import save_file

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(config, indent=1))
    save_file(tensors if tensors is not None else draw_tensors(config, seed, dtype, std), str(folder / "model.safetensors"))
    return folder


def read_model_dir(folder: Path) -> tuple[dict, dict[str, torch.Tensor]]:
    from safetensors.torch import load_file

    config = json.loads((Path(folder) / "config.json").read_text())
    tensors = {name: t.to(torch.float32) for name, t in load_file(str(Path(folder) / "model.safetensors")).items()}
    return config, tensors


def greedy(config: dict, tensors: dict[str, torch.Tensor], prompt: list[int], new: int) -> list[int]:
    tokens = list(prompt)
    for _ in range(new):
        tokens.append(int(plain.forward(config, tensors, tokens)[-1].argmax()))
    return tokens[len(prompt):]
