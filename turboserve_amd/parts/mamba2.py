"""Mamba-2: a mixer whose memory is one matrix per head and request, which every token decays by one number and
adds an outer product to."""

from __future__ import annotations

from collections.abc import Mapping

import torch

from turboserve_amd.parts.base import CacheNeed, FixedState, Mixer, Runtime, TensorSpec
from turboserve_amd.parts.registry import register_mixer


@register_mixer("mamba2")
class Mamba2(Mixer):
    """Per head a state ``S [N, P]`` (32-bit, zero when the request starts).  One matrix makes ``[z: H P | x: H P | B: G
    N | C: G N | d: H]`` of a token; ``x``, ``B`` and ``C`` pass a causal convolution over time of ``taps`` taps per channel
    with a bias and ``silu``; head ``h`` uses the ``B`` and ``C`` of group ``h // (H / G)``:

        dt = softplus(d + dt_bias_h)
        S <- exp(-exp(A_log_h) dt) S + dt B x^T;  y = S^T C + D_h x

    The heads' ``y`` side by side are multiplied by ``silu(z)``, each of ``norm_groups`` equal parts is divided by its
    own root mean square, and the whole, times a gain ``[H P]``, goes through the output matrix.  Everything that enters
    the recurrence behind the projection and the convolution is 32-bit.

    The state and the convolution's last ``taps - 1`` inputs are ``FixedState``s of the cache: the request's slot
    holds them between steps (the state with ``N`` innermost).  Single tokens, short portions and 32-bit runs walk each
    request's tokens in one launch; long portions are cut into pieces that run side by side on the matrix cores
    (``ops.selective_state``).  ``names``: tensor names under the part's prefix of ``in, conv, conv_bias, dt_bias, a_log,
    skip, norm, o``."""

    def __init__(self, prefix: str, runtime: Runtime, *, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int,
                 taps: int, norm_groups: int, norm_eps: float, names: Mapping[str, str] | None = None) -> None:
        super().__init__(prefix, runtime)
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.value_dim = int(value_dim)
        self.state_dim = int(state_dim)
        self.groups = int(groups)
        self.taps = int(taps)
        self.norm_groups = int(norm_groups)
        self.norm_eps = float(norm_eps)
        where = prefix or "mamba2"
        if min(self.num_heads, self.value_dim, self.state_dim, self.groups, self.norm_groups) < 1:
            raise ValueError(f"{where}: sizes must be positive")
        if self.num_heads % self.groups != 0:
            raise ValueError(f"{where}: {self.num_heads} heads are not a multiple of {self.groups} groups")
        self.inner = self.num_heads * self.value_dim
        if self.inner % self.norm_groups != 0:
            raise ValueError(f"{where}: {self.inner} channels are not {self.norm_groups} equal parts")
        if self.state_dim > 512 or self.num_heads > 65535 or self.inner // self.norm_groups > 16384:
            raise ValueError(f"{where}: the kernels take up to 512 state rows a head and parts of up to 16,384 channels")
        if not 1 <= self.taps <= 8:
            raise ValueError(f"{where}: a convolution of {self.taps} taps is outside 1..8")
        self.names = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "skip": "D",
                      "norm": "norm", "o": "o", **(names or {})}
        self.channels = self.inner + 2 * self.groups * self.state_dim  # what the convolution runs over
        self.rows = 2 * self.inner + 2 * self.groups * self.state_dim + self.num_heads
        self.in_weight: torch.Tensor | None = None    # [rows (padded), hidden]
        self.conv_weight: torch.Tensor | None = None  # [channels, taps]
        self.conv_bias: torch.Tensor | None = None    # [channels]
        self.dt_bias: torch.Tensor | None = None      # [H] 32-bit, as are a_log and skip
        self.a_log: torch.Tensor | None = None
        self.skip: torch.Tensor | None = None
        self.gain: torch.Tensor | None = None         # [H P]
        self.o_weight: torch.Tensor | None = None     # [hidden, H P]

    def cache_need(self) -> CacheNeed:
        return (FixedState((self.num_heads, self.value_dim, self.state_dim), torch.float32),
                FixedState((max(self.taps - 1, 1), self.channels), torch.float32))

    def activation_bytes(self, tokens: int, itemsize: int) -> int:
        pieces = -(-tokens // 128) + 1
        state = pieces * self.num_heads * (self.value_dim * self.state_dim + 1) * 4
        return tokens * ((self.rows + 16 + self.channels + self.inner) * itemsize + self.inner * 4 + self.hidden_size * 4) + state

    def tensor_specs(self) -> dict[str, TensorSpec]:
        n = self.names
        return {
            self.name(n["in"]): TensorSpec((self.rows, self.hidden_size)),
            self.name(n["conv"]): TensorSpec((self.channels, self.taps)),
            self.name(n["conv_bias"]): TensorSpec((self.channels,), init="zeros"),
            self.name(n["dt_bias"]): TensorSpec((self.num_heads,), kind="float_keep32", init="zeros"),
            self.name(n["a_log"]): TensorSpec((self.num_heads,), kind="float_keep32", init="zeros"),
            self.name(n["skip"]): TensorSpec((self.num_heads,), kind="float_keep32", init="ones"),
            self.name(n["norm"]): TensorSpec((self.inner,), init="ones"),
            self.name(n["o"]): TensorSpec((self.hidden_size, self.inner)),
        }

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        n = self.names
        weight = tensors[self.name(n["in"])]
        # Rows of zeros up to a multiple of 16: a row of the projection then starts on 16 bytes.
        padding = torch.zeros((-self.rows % 16, self.hidden_size), dtype=weight.dtype, device=weight.device)
        self.in_weight = torch.cat([weight, padding], dim=0).contiguous()
        del weight
        self.conv_weight = tensors[self.name(n["conv"])].contiguous()
        self.conv_bias = tensors[self.name(n["conv_bias"])].contiguous()
        self.dt_bias, self.a_log, self.skip = (tensors[self.name(n[key])].float().contiguous() for key in ("dt_bias", "a_log", "skip"))
        self.gain = tensors[self.name(n["norm"])].contiguous()
        self.o_weight = tensors[self.name(n["o"])].contiguous()

    def forward(self, x: torch.Tensor, ctx, cache) -> torch.Tensor:
        return self.runtime.ops.linear(self.heads_out(x, ctx, cache), self.o_weight, for_residual=True)

    def heads_out(self, x: torch.Tensor, ctx, cache) -> torch.Tensor:
        """Everything but the output matrix: ``[T, H P]`` of the run dtype."""
        ops, dtype = self.runtime.ops, self.runtime.dtype
        memory, held = cache
        proj = ops.linear(x, self.in_weight)
        u = ops.short_conv(proj, self.inner, self.conv_weight, held.state, ctx.state_slots, ctx.token_seq, ctx.query_start_loc,
                           tokens=ctx.num_tokens, num_seqs=ctx.num_seqs, dtype=dtype, silu=True, bias=self.conv_bias)
        plan = ops.decaying_plan(ctx, dtype, self.state_dim, self.value_dim)
        y = ops.selective_state(u, proj, self.inner + self.channels, self.dt_bias, self.a_log, self.skip, memory.state, ctx.state_slots,
                                ctx.query_start_loc, num_seqs=ctx.num_seqs, heads=self.num_heads, groups=self.groups,
                                state_dim=self.state_dim, value_dim=self.value_dim, dtype=dtype, plan=plan)
        return ops.gated_group_norm(y, proj, 0, self.gain, self.norm_eps, self.norm_groups, dtype)
