"""Small Lukelix configurations that differ in every size, constant and layer order, and helpers that
write their random model folders and compute the plain implementation's logits."""

from __future__ import annotations

import json
from pathlib import Path

import torch

from plain import lukelix_plain as plain


def attention(heads, kv_heads, dim, vdim=None, conv=None, scale=None, rot=None, bands=None, base=10000.0, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim if vdim is None else vdim,
             "scale": dim ** -0.5 if scale is None else scale}
    if conv is not None:
        mixer["conv"] = conv
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    if rot is not None:
        mixer["rot"] = {"base": base, "dims": rot}
        if bands is not None:
            mixer["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), bands))
    return {"type": "attention", "mixer": mixer}


def mamba2(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}}


def layer(mixer, ff=None):
    return {**mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def bigram(buckets, mul_prev, mul_cur):
    return {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}


#: A: state layers first, one with a feed-forward; attention without one; a layer that reads the keys of one two
#: layers back, with other convolution taps and a scale of its own; a head rotated in part with wavelengths in all
#: three bands; values wider than keys.
CONFIG_A = {
    "architecture": "Lukelix", "vocab": 211, "width": 64, "norm": {"eps": 1e-5}, "embedding": bigram(97, 13, 5),
    "layers": [
        layer(mamba2(4, 16, 24, 2, 4, 2), 40),
        layer(attention(4, 2, 16, 24, conv=3, scale=0.3, rot=8, bands=(4.0, 1.0, 4.0, 64), base=1000.0)),
        layer(mamba2(6, 8, 40, 3, 2, 1)),
        layer(attention(4, 2, 16, 24, conv=2, scale=0.5, rot=8, bands=(4.0, 1.0, 4.0, 64), base=1000.0, kv_from=1), 96),
        layer(mamba2(2, 40, 8, 1, 3, 5)),
    ],
}
PAGE_A = 16

#: B: sizes that 16-byte accesses do not divide; one head; as many key heads as query heads; attention without a
#: convolution, without a rotation, with one tap; one state row; one bucket; a table with multipliers beyond it; two
#: layers that read one layer's keys.
CONFIG_B = {
    "architecture": "Lukelix", "vocab": 97, "width": 51, "norm": {"eps": 1e-6}, "embedding": bigram(31, 1000003, 37),
    "layers": [
        layer(attention(3, 3, 12, scale=0.4, rot=12, base=50.0), 28),
        layer(attention(3, 3, 12, conv=1, scale=0.7, rot=12, base=50.0, kv_from=0)),
        layer(mamba2(1, 20, 1, 1, 1, 1), 20),
        layer(attention(1, 1, 20, 7, conv=5)),
        layer(mamba2(5, 6, 33, 5, 8, 3)),
        layer(attention(6, 3, 12, conv=4, rot=2, bands=(2.0, 0.5, 2.0, 16), kv_from=0), 12),
    ],
}
PAGE_B = 8

#: C: heads on the matrix-core path, state rows and columns on the path that cuts portions into pieces, pages of 32,
#: no bigram table.
CONFIG_C = {
    "architecture": "Lukelix", "vocab": 160, "width": 96, "norm": {"eps": 1e-6},
    "layers": [
        layer(attention(6, 2, 32, conv=4, scale=0.25, rot=32, bands=(6.0, 1.0, 3.0, 128), base=200000.0), 48),
        layer(mamba2(4, 32, 64, 2, 4, 4)),
        layer(attention(6, 2, 32, conv=3, rot=32, bands=(6.0, 1.0, 3.0, 128), base=200000.0, kv_from=0)),
        layer(mamba2(8, 8, 136, 4, 3, 2), 64),
        layer(attention(8, 1, 64, rot=16)),
    ],
}
PAGE_C = 32

TINY = {"A": (CONFIG_A, 31, PAGE_A), "B": (CONFIG_B, 32, PAGE_B), "C": (CONFIG_C, 33, PAGE_C)}


def draw_tensors(config: dict, seed: int, dtype: torch.dtype, std: float) -> dict[str, torch.Tensor]:
    """Random tensors by the names and shapes the engine's own description of the model gives (the plain
    implementation reads them by name): matrices N(0, std); norm weights around one; convolution taps, biases and decay
    rates wide enough to matter (decays from a few tokens to hundreds)."""
    from turboserve_amd.weights.random_init import describe_model

    _, model = describe_model(config)
    generator = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, spec in model.tensor_specs().items():
        values = torch.randn(spec.shape, generator=generator)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm", "norm1", "norm2"):
            values = 1.0 + 0.3 * values
        elif leaf == "b":
            values = 0.3 * values
        elif name in ("embed", "bigram"):
            values = 0.7 * values
        elif leaf == "conv":
            values = 0.6 * values
        elif leaf == "A_log":
            values = -1.0 + 1.5 * values
        elif leaf == "dt_bias":
            values = -1.5 + values
        elif leaf == "D":
            values = 0.5 + 0.5 * values
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


def plain_logits(folder: Path, tokens: list[int]) -> torch.Tensor:
    config, tensors = read_model_dir(folder)
    return plain.forward(config, tensors, tokens)


def greedy(config: dict, tensors: dict[str, torch.Tensor], prompt: list[int], new: int) -> list[int]:
    tokens = list(prompt)
    for _ in range(new):
        tokens.append(int(plain.forward(config, tensors, tokens)[-1].argmax()))
    return tokens[len(prompt):]
