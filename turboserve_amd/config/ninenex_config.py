"""Typed view of a Ninenex ``config.json``.

The file names the design under ``architecture`` and describes every layer on its own::

    {"architecture": "Ninenex", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s}, "logit_scale": z,
     "layers": [{"type": "mlstm", "mixer": {"heads": H, "dim": D, "vdim": Dv, "gate_cap": c}, "mlp": ...},
                {"type": "parallel",
                 "mixer": {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": s, "mask": {"size": C},
                                    "rot": {"base": b, "dims": d}},
                           "right": {"heads": H, "dim": D, "vdim": Dv, "decay": [d_0, ..]},
                           "left_scale": a, "right_scale": b},
                 "mlp": null
                      | {"kind": "dense", "ff": I}
                      | {"kind": "moe", "expert": {"ff": I}, "router": {"experts": E, "top": k}, "shared": {"ff": J} | null},
                 "weights_of": j}, ...]}

Every size and constant a model of the design can choose comes from here; what is absent or null (a mask, a rotation, a
feed-forward, a shared expert) does not exist in that model.  A layer with ``weights_of`` runs with layer ``j``'s tensors
and a cache or state of its own; the rest of its entry is layer ``j``'s.  What the design fixes lives where the plan is
put together.
"""

from __future__ import annotations

from collections.abc import Mapping
from dataclasses import dataclass
from typing import Any

from turboserve_amd.config.model_config import UnsupportedModelError
from turboserve_amd.config.sisisun_config import _count, _mapping, _real

ARCHITECTURE = "Ninenex"
MIXER_TYPES = ("mlstm", "parallel")


def _optional(where: str, data: Mapping[str, Any], key: str) -> Mapping[str, Any] | None:
    return None if data.get(key) is None else _mapping(where, data, key)


@dataclass(frozen=True)
class MatrixMemorySizes:
    """A matrix memory with exponential gates."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "MatrixMemorySizes":
        return cls(_count(where, data, "heads"), _count(where, data, "dim"), _count(where, data, "vdim"), _real(where, data, "gate_cap"))

    def cached_elements(self) -> int:
        return 0


@dataclass(frozen=True)
class ChunkedAttentionSizes:
    """The left mixer of a parallel layer: biased projections, rotation of a head's first elements, chunks."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int | None
    rot_base: float | None
    rot_dims: int

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "ChunkedAttentionSizes":
        heads, kv_heads, dim = _count(where, data, "heads"), _count(where, data, "kv_heads"), _count(where, data, "dim")
        if heads % kv_heads != 0:
            raise UnsupportedModelError(f"config.json: {where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        mask, rot = _optional(where, data, "mask"), _optional(where, data, "rot")
        chunk = None if mask is None else _count(f"{where}.mask", mask, "size")
        base, dims = None, 0
        if rot is not None:
            base, dims = _real(f"{where}.rot", rot, "base"), _count(f"{where}.rot", rot, "dims", least=2)
            if dims > dim or dims % 2 != 0:
                raise UnsupportedModelError(f"config.json: {where}.rot.dims {dims} must be even and at most dim {dim}")
        return cls(heads, kv_heads, dim, _count(where, data, "vdim"), _real(where, data, "scale"), chunk, base, dims)


@dataclass(frozen=True)
class RetentionSizes:
    """The right mixer of a parallel layer: linear attention with a fixed decay per head."""

    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "RetentionSizes":
        heads, listed = _count(where, data, "heads"), data.get("decay")
        numbers = isinstance(listed, (list, tuple)) and all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in listed)
        if not numbers or len(listed) != heads or not all(0.0 < d <= 1.0 for d in listed):
            raise UnsupportedModelError(f"config.json: {where}.decay must list a number above 0 and at most 1 for each of {heads} heads, "
                                        f"got {listed!r}")
        return cls(heads, _count(where, data, "dim"), _count(where, data, "vdim"), tuple(float(d) for d in listed))


@dataclass(frozen=True)
class ParallelSizes:
    left: ChunkedAttentionSizes
    right: RetentionSizes
    left_scale: float
    right_scale: float

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "ParallelSizes":
        return cls(ChunkedAttentionSizes.read(f"{where}.left", _mapping(where, data, "left")),
                   RetentionSizes.read(f"{where}.right", _mapping(where, data, "right")),
                   _real(where, data, "left_scale", positive=False), _real(where, data, "right_scale", positive=False))

    def cached_elements(self) -> int:
        return self.left.kv_heads * (self.left.dim + self.left.vdim)


@dataclass(frozen=True)
class DenseSizes:
    ff: int


@dataclass(frozen=True)
class RoutedSizes:
    ff: int
    experts: int
    top: int
    shared_ff: int  # 0: no shared expert


def _feed_forward(where: str, data: Mapping[str, Any]) -> DenseSizes | RoutedSizes:
    kind = data.get("kind")
    if kind == "dense":
        return DenseSizes(_count(where, data, "ff"))
    if kind != "moe":
        raise UnsupportedModelError(f"config.json: {where}.kind {kind!r} is not implemented; supported: ['dense', 'moe']")
    router, shared = _mapping(where, data, "router"), _optional(where, data, "shared")
    sizes = RoutedSizes(
        ff=_count(f"{where}.expert", _mapping(where, data, "expert"), "ff"), experts=_count(f"{where}.router", router, "experts"),
        top=_count(f"{where}.router", router, "top"), shared_ff=0 if shared is None else _count(f"{where}.shared", shared, "ff"))
    if sizes.top > sizes.experts:
        raise UnsupportedModelError(f"config.json: {where}.router: top {sizes.top} of {sizes.experts} experts")
    return sizes


@dataclass(frozen=True)
class NinenexLayer:
    type: str
    mixer: MatrixMemorySizes | ParallelSizes
    mlp: DenseSizes | RoutedSizes | None
    weights_of: int  # the layer whose tensors this one uses (its own index: its own)


@dataclass(frozen=True)
class NinenexConfig:
    """One checkpoint's numbers (frozen: model, cache sizing and runner share it)."""

    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    layers: tuple[NinenexLayer, ...]
    eos_token_ids: tuple[int, ...] = ()
    name_or_path: str = ""

    def kv_bytes_per_token(self, dtype) -> int:
        """Bytes one token takes in the pages of all layers (each has pages of its own, also one that runs with another's
        tensors)."""
        return sum(layer.mixer.cached_elements() for layer in self.layers) * dtype.itemsize

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], *, name_or_path: str = "") -> "NinenexConfig":
        if str(data.get("architecture")) != ARCHITECTURE:
            raise UnsupportedModelError(f"architecture {data.get('architecture')!r} is not {ARCHITECTURE}")
        listed = data.get("layers")
        if not isinstance(listed, (list, tuple)) or not listed:
            raise UnsupportedModelError("config.json: layers must be a non-empty list")
        readers = {"mlstm": MatrixMemorySizes, "parallel": ParallelSizes}
        layers = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            if not isinstance(entry, Mapping):
                raise UnsupportedModelError(f"config.json: {where} must be an object")
            kind = entry.get("type")
            if kind not in readers:
                raise UnsupportedModelError(f"config.json: {where}.type {kind!r} is not implemented; supported: {list(MIXER_TYPES)}")
            mixer = readers[kind].read(f"{where}.mixer", _mapping(where, entry, "mixer"))
            mlp = None if entry.get("mlp") is None else _feed_forward(f"{where}.mlp", _mapping(where, entry, "mlp"))
            layers.append(NinenexLayer(kind, mixer, mlp, cls._owner(listed, index)))
        for index, layer in enumerate(layers):
            owner = layers[layer.weights_of]
            if (layer.type, layer.mixer, layer.mlp) != (owner.type, owner.mixer, owner.mlp):
                raise UnsupportedModelError(f"config.json: layers[{index}].weights_of: the entry differs from layer {layer.weights_of}'s")
        named = data.get("eos_token_id")
        eos = () if named is None else (int(named),) if isinstance(named, int) else tuple(int(t) for t in named)
        embedding = _optional("config", data, "embedding") or {}
        return cls(
            architecture=ARCHITECTURE, vocab_size=_count("config", data, "vocab"), hidden_size=_count("config", data, "width"),
            norm_eps=_real("norm", _mapping("config", data, "norm"), "eps"),
            embedding_scale=1.0 if embedding.get("scale") is None else _real("embedding", embedding, "scale", positive=False),
            logit_scale=1.0 if data.get("logit_scale") is None else _real("config", data, "logit_scale", positive=False),
            layers=tuple(layers), eos_token_ids=eos, name_or_path=name_or_path,
        )

    @staticmethod
    def _owner(listed, index: int) -> int:
        """The layer whose tensors layer ``index`` uses, through layers that themselves use another's."""
        passed = []
        while isinstance(listed[index], Mapping) and listed[index].get("weights_of") is not None:
            passed.append(index)
            where = f"layers[{index}]"
            index = _count(where, listed[index], "weights_of", least=0)
            if index >= len(listed) or index in passed:
                raise UnsupportedModelError(f"config.json: {where}.weights_of {index} names no layer with tensors of its own")
        return index
