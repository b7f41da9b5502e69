"""Typed view of a Lukelix ``config.json``.

The file names the design under ``architecture`` and describes every layer on its own::

    {"architecture": "Lukelix", "vocab": V, "width": W, "norm": {"eps": e},
     "embedding": {"bigram": {"buckets": n, "mul_prev": a, "mul_cur": b}},
     "layers": [{"type": "attention",
                 "mixer": {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": s, "conv": K, "kv_from": j,
                           "rot": {"base": b, "dims": d,
                                   "scaling": {"factor": f, "low": l, "high": h, "original": n}}},
                 "mlp": {"kind": "dense", "ff": I} | null},
                {"type": "mamba2",
                 "mixer": {"heads": H, "vdim": P, "state": N, "groups": G, "conv": K, "norm_groups": n},
                 "mlp": ...}, ...]}

Every size and constant a model of the design can choose comes from here; what is absent or null (the bigram
table, a convolution of an attention layer, another layer's keys, a rotation or its scaling, a feed-forward) does not
exist in that model.  What the design fixes lives where the plan is put together.
"""

from __future__ import annotations

from collections.abc import Mapping
from dataclasses import dataclass
from typing import Any

from turboserve_amd.config.model_config import UnsupportedModelError
from turboserve_amd.config.sisisun_config import _count, _mapping, _real

ARCHITECTURE = "Lukelix"
MIXER_TYPES = ("attention", "mamba2")


@dataclass(frozen=True)
class BandScaling:
    """Long wavelengths of a rotation stretched: kept below ``original / high``, divided by ``factor`` above
    ``original / low``, blended between."""

    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "BandScaling":
        return cls(*(_real(where, data, key) for key in ("factor", "low", "high", "original")))

    def as_mapping(self) -> dict[str, float]:
        return {"factor": self.factor, "low": self.low, "high": self.high, "original": self.original}


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    taps: int | None
    kv_from: int | None  # the layer whose keys and values this one reads
    rot_base: float | None
    rot_dims: int
    rot_scaling: BandScaling | None

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "AttentionSizes":
        heads, kv_heads = _count(where, data, "heads"), _count(where, data, "kv_heads")
        if heads % kv_heads != 0:
            raise UnsupportedModelError(f"config.json: {where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        dim = _count(where, data, "dim")
        base, dims, scaling = None, 0, None
        if data.get("rot") is not None:
            rot = _mapping(where, data, "rot")
            base, dims = _real(f"{where}.rot", rot, "base"), _count(f"{where}.rot", rot, "dims", least=2)
            if dims > dim or dims % 2 != 0:
                raise UnsupportedModelError(f"config.json: {where}.rot.dims {dims} must be even and at most dim {dim}")
            if rot.get("scaling") is not None:
                scaling = BandScaling.read(f"{where}.rot.scaling", _mapping(f"{where}.rot", rot, "scaling"))
        return cls(heads, kv_heads, dim, _count(where, data, "vdim"), _real(where, data, "scale"),
                   None if data.get("conv") is None else _count(where, data, "conv"),
                   None if data.get("kv_from") is None else _count(where, data, "kv_from", least=0), base, dims, scaling)

    def cached_elements(self) -> int:
        return 0 if self.kv_from is not None else self.kv_heads * (self.dim + self.vdim)


@dataclass(frozen=True)
class Mamba2Sizes:
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "Mamba2Sizes":
        sizes = cls(*(_count(where, data, key) for key in ("heads", "vdim", "state", "groups", "conv", "norm_groups")))
        if sizes.heads % sizes.groups != 0:
            raise UnsupportedModelError(f"config.json: {where}: {sizes.heads} heads are not a multiple of {sizes.groups} groups")
        if (sizes.heads * sizes.vdim) % sizes.norm_groups != 0:
            raise UnsupportedModelError(f"config.json: {where}: {sizes.heads * sizes.vdim} channels are not {sizes.norm_groups} equal norm_groups")
        return sizes

    def cached_elements(self) -> int:
        return 0


@dataclass(frozen=True)
class BigramRule:
    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def read(cls, where: str, data: Mapping[str, Any]) -> "BigramRule":
        return cls(_count(where, data, "buckets"), *(_count(where, data, key, least=0) for key in ("mul_prev", "mul_cur")))


@dataclass(frozen=True)
class LukelixLayer:
    type: str
    mixer: AttentionSizes | Mamba2Sizes
    ff: int | None


@dataclass(frozen=True)
class LukelixConfig:
    """One checkpoint's numbers (frozen: model, cache sizing and runner share it)."""

    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    bigram: BigramRule | None
    layers: tuple[LukelixLayer, ...]
    eos_token_ids: tuple[int, ...] = ()
    name_or_path: str = ""

    def kv_bytes_per_token(self, dtype) -> int:
        """Bytes one token takes in the pages of all layers."""
        return sum(layer.mixer.cached_elements() for layer in self.layers) * dtype.itemsize

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], *, name_or_path: str = "") -> "LukelixConfig":
        if str(data.get("architecture")) != ARCHITECTURE:
            raise UnsupportedModelError(f"architecture {data.get('architecture')!r} is not {ARCHITECTURE}")
        listed = data.get("layers")
        if not isinstance(listed, (list, tuple)) or not listed:
            raise UnsupportedModelError("config.json: layers must be a non-empty list")
        readers = {"attention": AttentionSizes, "mamba2": Mamba2Sizes}
        layers: list[LukelixLayer] = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            if not isinstance(entry, Mapping):
                raise UnsupportedModelError(f"config.json: {where} must be an object")
            kind = entry.get("type")
            if kind not in readers:
                raise UnsupportedModelError(f"config.json: {where}.type {kind!r} is not implemented; supported: {list(MIXER_TYPES)}")
            mixer = readers[kind].read(f"{where}.mixer", _mapping(where, entry, "mixer"))
            _check_source(where, mixer, layers)
            ff = None
            if entry.get("mlp") is not None:
                mlp = _mapping(where, entry, "mlp")
                if mlp.get("kind") != "dense":
                    raise UnsupportedModelError(f"config.json: {where}.mlp.kind {mlp.get('kind')!r} is not implemented; supported: ['dense']")
                ff = _count(f"{where}.mlp", mlp, "ff")
            layers.append(LukelixLayer(kind, mixer, ff))
        embedding = {} if data.get("embedding") is None else _mapping("config", data, "embedding")
        bigram = None
        if embedding.get("bigram") is not None:
            bigram = BigramRule.read("embedding.bigram", _mapping("embedding", embedding, "bigram"))
        named = data.get("eos_token_id")
        eos = () if named is None else (int(named),) if isinstance(named, int) else tuple(int(t) for t in named)
        return cls(
            architecture=ARCHITECTURE, vocab_size=_count("config", data, "vocab"), hidden_size=_count("config", data, "width"),
            norm_eps=_real("norm", _mapping("config", data, "norm"), "eps"), bigram=bigram, layers=tuple(layers),
            eos_token_ids=eos, name_or_path=name_or_path,
        )


def _check_source(where: str, mixer, layers: list[LukelixLayer]) -> None:
    """``kv_from`` names an earlier attention layer with keys of its own and the same cached sizes."""
    source = getattr(mixer, "kv_from", None)
    if source is None:
        return
    other = layers[source].mixer if source < len(layers) else None
    if not isinstance(other, AttentionSizes) or other.kv_from is not None:
        raise UnsupportedModelError(f"config.json: {where}.mixer.kv_from {source} is not an earlier attention layer with keys of its own")
    if (other.kv_heads, other.dim, other.vdim) != (mixer.kv_heads, mixer.dim, mixer.vdim):
        raise UnsupportedModelError(f"config.json: {where}.mixer.kv_from: layer {source} keeps {other.kv_heads} heads of {other.dim}/{other.vdim}, "
                                    f"this layer reads {mixer.kv_heads} of {mixer.dim}/{mixer.vdim}")
