"""Mixers whose memory is one matrix per head and request that decays by one number per head and token:
retention (a fixed decay) and the matrix memory of xLSTM (exponential gates)."""

from __future__ import annotations

from collections.abc import Mapping, Sequence

import torch

from turboserve_amd.parts.base import CacheNeed, FixedState, Mixer, Runtime, TensorSpec
from turboserve_amd.parts.registry import register_mixer


class DecayingMemory(Mixer):
    """What the mixers below have in common.  Per head a state ``S [D, Dv]`` (32-bit, zero when the request starts) takes
    every token as ``S <- a S + w k v^T`` and is read as ``S^T q``, with ``q = Wq x``, ``k = Wk x``, ``v = Wv x``; how ``a``
    and ``w`` are made is the mixer's.  A head's read-out is divided by its root mean square, the heads side by side are
    multiplied by a gate made from ``Wg x`` and go through the output matrix.

    ``Wq, Wk, Wv, Wg`` and the mixer's own rows are held as one matrix (one product a step).  The state is a ``FixedState``
    of the cache (with ``D`` innermost).  Single tokens, short portions and 32-bit runs walk each request's tokens in one
    launch; long portions are cut into pieces that run side by side on the matrix cores (``ops.decaying_state``)."""

    o_bias_tensor = None

    def __init__(self, prefix: str, runtime: Runtime, what: str, *, hidden_size: int, num_heads: int, head_dim: int, value_dim: int,
                 norm_eps: float, names: Mapping[str, str]) -> None:
        super().__init__(prefix, runtime)
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.head_dim = int(head_dim)
        self.value_dim = int(value_dim)
        self.norm_eps = float(norm_eps)
        self.names = dict(names)
        self.where = prefix or what
        if min(self.num_heads, self.head_dim, self.value_dim) < 1:
            raise ValueError(f"{self.where}: sizes must be positive")
        if self.head_dim > 512 or self.num_heads > 65535 or self.value_dim > 65534:
            raise ValueError(f"{self.where}: the kernels take up to 512 key channels a head")
        self.key_size = self.num_heads * self.head_dim
        self.value_size = self.num_heads * self.value_dim
        self.gate_at = 2 * self.key_size + self.value_size   # the gate's first column of the fused projection
        self.more_at = self.gate_at + self.value_size        # the mixer's own columns
        self.fused: torch.Tensor | None = None      # [2 H D + 2 H Dv + .. (padded), hidden]
        self.o_weight: torch.Tensor | None = None   # [hidden, H Dv]

    #: Rows of the fused matrix behind q, k, v and the gate, by tensor.
    more_rows: Sequence[str] = ()

    def state_needs(self) -> tuple[FixedState, ...]:
        return (FixedState((self.num_heads, self.value_dim, self.head_dim), torch.float32),)

    def cache_need(self) -> CacheNeed:
        needs = self.state_needs()
        return needs[0] if len(needs) == 1 else needs

    def activation_bytes(self, tokens: int, itemsize: int) -> int:
        pieces = -(-tokens // 128) + 1
        state = pieces * self.num_heads * (self.value_dim + 1) * (self.head_dim + 4) * 4
        rows = self.more_at + len(self.more_rows) * self.num_heads + 16
        return tokens * ((rows + self.value_size) * itemsize + (self.value_size + 2 * self.num_heads + self.hidden_size) * 4) + state

    def tensor_specs(self) -> dict[str, TensorSpec]:
        sizes = {"q": self.key_size, "k": self.key_size, "v": self.value_size, "gate": self.value_size}
        sizes.update({which: self.num_heads for which in self.more_rows})
        specs = {self.name(self.names[which]): TensorSpec((rows, self.hidden_size)) for which, rows in sizes.items()}
        specs[self.name(self.names["o"])] = TensorSpec((self.hidden_size, self.value_size))
        return specs

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        rows = [tensors[self.name(self.names[which])] for which in ("q", "k", "v", "gate", *self.more_rows)]
        # Rows of zeros up to a multiple of 16: a row of the projection then starts on 16 bytes.
        padding = -sum(r.shape[0] for r in rows) % 16
        rows.append(torch.zeros((padding, self.hidden_size), dtype=rows[0].dtype, device=rows[0].device))
        self.fused = torch.cat(rows, dim=0).contiguous()
        del rows
        self.o_weight = tensors[self.name(self.names["o"])].contiguous()

    @property
    def out_features(self) -> int:
        """The width of what the output matrix multiplies."""
        return self.value_size

    def scales_its_heads(self) -> bool:
        return True

    def forward(self, x: torch.Tensor, ctx, cache) -> torch.Tensor:
        return self.runtime.ops.linear(self.heads_out(x, ctx, cache), self.o_weight, for_residual=True)

    def heads_out(self, x: torch.Tensor, ctx, cache, *, scale: float = 1.0, out: tuple | None = None) -> torch.Tensor:
        """Everything but the output matrix: ``[T, H Dv]`` of the run dtype times ``scale``, optionally written into
        columns of a wider buffer (``out = (buffer, col0)``)."""
        raise NotImplementedError

    def _walk(self, rule: str, rows: torch.Tensor, ctx, memory, **more):
        """The recurrence over the step; read-outs carry the factor ``D^-1/2`` that belongs to the query or the key."""
        ops, dtype = self.runtime.ops, self.runtime.dtype
        return ops.decaying_state(
            rule, rows, (2 * self.key_size, self.key_size, 0), memory.state, ctx.state_slots, ctx.query_start_loc, num_seqs=ctx.num_seqs,
            heads=self.num_heads, groups=self.num_heads, state_dim=self.head_dim, value_dim=self.value_dim, dtype=dtype,
            scale=self.head_dim ** -0.5, plan=ops.decaying_plan(ctx, dtype, self.head_dim, self.value_dim), **more)


@register_mixer("retention")
class Retention(DecayingMemory):
    """Linear attention with a fixed decay per head and no denominator: ``S <- decay_h S + k v^T``, ``o = D^-1/2 S^T q``;
    a head's ``o`` is divided by its root mean square (no gain) and multiplied by ``silu(Wg x)``.  ``decay``: one number
    per head, above 0 and at most 1.  ``names``: tensor names under the part's prefix of ``q, k, v, gate, o``."""

    def __init__(self, prefix: str, runtime: Runtime, *, hidden_size: int, num_heads: int, head_dim: int, value_dim: int,
                 decay: Sequence[float], norm_eps: float, names: Mapping[str, str] | None = None) -> None:
        super().__init__(prefix, runtime, "retention", hidden_size=hidden_size, num_heads=num_heads, head_dim=head_dim,
                         value_dim=value_dim, norm_eps=norm_eps,
                         names={"q": "q", "k": "k", "v": "v", "gate": "g", "o": "o", **(names or {})})
        self.decay = tuple(float(d) for d in decay)
        if len(self.decay) != self.num_heads or not all(0.0 < d <= 1.0 for d in self.decay):
            raise ValueError(f"{self.where}: a decay above 0 and at most 1 for each of {self.num_heads} heads, not {list(decay)}")
        self.decays: torch.Tensor | None = None  # [H] 32-bit

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        super().load(tensors)
        self.decays = torch.tensor(self.decay, dtype=torch.float32, device=self.fused.device)

    def heads_out(self, x: torch.Tensor, ctx, cache, *, scale: float = 1.0, out: tuple | None = None) -> torch.Tensor:
        ops, dtype = self.runtime.ops, self.runtime.dtype
        proj = ops.linear(x, self.fused)
        y, _ = self._walk("fixed", proj, ctx, cache, numbers=(self.decays,))
        return ops.heads_finish(y, proj, self.gate_at, self.num_heads, self.norm_eps, dtype, gate="silu", scale=scale, out=out)


@register_mixer("mlstm")
class MatrixMemory(DecayingMemory):
    """The matrix memory of xLSTM.  Per head a log input gate ``i = cap tanh((Wi x + bi) / cap)`` and a log forget gate ``f =
    log sigmoid(cap tanh((Wf x + bf) / cap))``; with a running maximum ``m`` that starts at 0, ``m' = max(f + m, i)``, the
    state and a sum ``n`` of keys decay by ``exp(f + m - m')`` and take the token with the weight ``exp(i - m')``; ``o = S^T q
    / (max(|n . q|, exp(-m')) + 1e-6)`` with ``q = D^-1/2 Wq x``.  A head's ``o`` is divided by its root mean square; the heads
    side by side are multiplied by a gain ``[H Dv]`` and by ``sigmoid(Wg x)``.  Everything that enters the recurrence
    behind the projection is 32-bit.

    Three ``FixedState``s: ``S``, ``n`` and ``m``.  ``names``: tensor names under the part's prefix of ``q, k, v, gate, in,
    forget, in_bias, forget_bias, norm, o``."""

    more_rows = ("in", "forget")

    def __init__(self, prefix: str, runtime: Runtime, *, hidden_size: int, num_heads: int, head_dim: int, value_dim: int,
                 gate_cap: float, norm_eps: float, names: Mapping[str, str] | None = None) -> None:
        super().__init__(prefix, runtime, "matrix memory", hidden_size=hidden_size, num_heads=num_heads, head_dim=head_dim,
                         value_dim=value_dim, norm_eps=norm_eps,
                         names={"q": "q", "k": "k", "v": "v", "gate": "g", "in": "i", "forget": "f", "in_bias": "i.b",
                                "forget_bias": "f.b", "norm": "norm", "o": "o", **(names or {})})
        self.gate_cap = float(gate_cap)
        if not self.gate_cap > 0.0:
            raise ValueError(f"{self.where}: a gate cap of {gate_cap}")
        self.in_bias: torch.Tensor | None = None      # [H] 32-bit, as is forget_bias
        self.forget_bias: torch.Tensor | None = None
        self.gain: torch.Tensor | None = None         # [H Dv]

    def state_needs(self) -> tuple[FixedState, ...]:
        return (*super().state_needs(), FixedState((self.num_heads, self.head_dim), torch.float32),
                FixedState((self.num_heads,), torch.float32))

    def tensor_specs(self) -> dict[str, TensorSpec]:
        n = self.names
        return {
            **super().tensor_specs(),
            self.name(n["in_bias"]): TensorSpec((self.num_heads,), kind="float_keep32", init="zeros"),
            self.name(n["forget_bias"]): TensorSpec((self.num_heads,), kind="float_keep32", init="zeros"),
            self.name(n["norm"]): TensorSpec((self.value_size,), init="ones"),
        }

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        super().load(tensors)
        self.in_bias, self.forget_bias = (tensors[self.name(self.names[key])].float().contiguous() for key in ("in_bias", "forget_bias"))
        self.gain = tensors[self.name(self.names["norm"])].contiguous()

    def heads_out(self, x: torch.Tensor, ctx, cache, *, scale: float = 1.0, out: tuple | None = None) -> torch.Tensor:
        ops, dtype = self.runtime.ops, self.runtime.dtype
        memory, sums, tops = cache
        proj = ops.linear(x, self.fused)
        y, norm = self._walk("gated", proj, ctx, memory, proj=proj, first_gate=self.more_at, numbers=(self.in_bias, self.forget_bias),
                             cap=self.gate_cap, sums=sums.state, tops=tops.state)
        return ops.heads_finish(y, proj, self.gate_at, self.num_heads, self.norm_eps, dtype, gate="sigmoid", gain=self.gain, norm=norm,
                                tops=tops.state, state_slots=ctx.state_slots, token_seq=ctx.token_seq,
                                query_start_loc=ctx.query_start_loc, scale=scale, out=out)
