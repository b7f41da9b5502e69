"""Ninenex on the GPU against the plain implementation (``tests/plain/ninenex_plain.py``): each mechanism
alone (its kernel, and a one-layer model of it), whole prompts, every way of cutting requests into steps
on so few pages and slots that they are used again, keys just inside and just outside a chunk, state that has
to last, and greedy generation through the engine's own entry point."""

from __future__ import annotations

import json
import random
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import ninenex_tiny as nt
import trace_helpers as th
from plain import ninenex_plain as plain

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
ROOT = Path(__file__).resolve().parent.parent
#: How far a position's logits may be off, relative to its largest (at least 1): the engine's 32-bit runs and its bfloat16
#: runs (weights stored in bfloat16) against the plain implementation in 64-bit on the same weights ...
FLOOR = {"float32": 1e-4, "bfloat16": 4e-2}
#: ... or this many times what changing every weight by a relative error of the run's rounding does to that position, where
#: that is more: norms behind parts and heads make a position whose output is small against its terms answer rounding
#: strongly.  In bfloat16 runs one position in twenty may be off by four times its bound (rounding can hand a token to
#: another expert where two router scores are close).
ANSWER = 4.0
ROUNDING = {"float32": 2.0 ** -22, "bfloat16": 2.0 ** -9}
BF16_OUTLIERS = 4.0


@pytest.fixture(scope="module")
def ops():
    from turboserve_amd.kernels.ops import Ops

    return Ops(DEV)


def expect(folder, tokens: list[int], dtype: str) -> tuple[torch.Tensor, torch.Tensor]:
    """The plain implementation's logits ``[T, V]`` in 64-bit and each position's bound ``[T]``."""
    raw, tensors = nt.read_model_dir(folder)
    tensors = {name: t.double() for name, t in tensors.items()}
    want = plain.forward(raw, tensors, tokens)
    bound = FLOOR[dtype] * want.abs().amax(dim=-1).clamp_min(1.0)
    for seed in (1, 2):
        g = torch.Generator().manual_seed(seed)
        off = {name: t * (1.0 + ROUNDING[dtype] * torch.randn(t.shape, generator=g).double()) for name, t in tensors.items()}
        bound = torch.maximum(bound, ANSWER * (plain.forward(raw, off, tokens) - want).abs().amax(dim=-1))
    return want, bound


def excess(got: torch.Tensor, expected: tuple[torch.Tensor, torch.Tensor], dtype: str) -> float:
    """The largest multiple of its bound that a position is off by (bfloat16: of nineteen positions in twenty; the rest count a
    quarter)."""
    want, bound = expected
    rows = ((got.double() - want).abs().amax(dim=-1) / bound).sort().values
    if dtype == "float32":
        return float(rows[-1])
    return max(float(rows[int(0.95 * (len(rows) - 1))]), float(rows[-1]) / BF16_OUTLIERS)


def tokens_of(vocab: int, length: int, seed: int) -> list[int]:
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (length,), generator=g).tolist()


def stored_as(dtype: str) -> torch.dtype:
    return torch.float32 if dtype == "float32" else torch.bfloat16


def run_trace(folder, dtype: str, page: int, steps: list[dict], max_tokens: int | None = None, max_live: int = 4):
    from turboserve_amd.engine.replay import TraceReplayer

    replayer = TraceReplayer(folder, dtype=dtype, max_tokens=max_tokens or th.peak_tokens(steps, rounding=page),
                             page_size=page, max_live=max_live)
    outputs = {}
    for record in steps:
        logits = replayer.run_step(record)
        if logits.shape[0]:
            outputs[record["step"]] = logits.float().cpu()
    replayer.manager.check_invariants()
    assert all(pool.num_in_use == 0 for pool in replayer.manager.pools), "pages were not given back"
    return outputs


def near(got: torch.Tensor, want: torch.Tensor, dtype: torch.dtype, loose: float = 1.0) -> None:
    tol = (2e-5 if dtype == torch.float32 else 1.6e-2) * loose
    scale = float(want.abs().max().clamp_min(1e-3))
    off = float((got.double().cpu() - want.double()).abs().max())
    assert off <= tol * scale, off / scale


def ints(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ---------------------------------------------------------------------------------------------
# mechanisms alone: the recurrences
# ---------------------------------------------------------------------------------------------

LENGTHS, SLOTS = [300, 129, 31], [3, 1, 4]


def walked(ops, rows: list[torch.Tensor], step, pieces: bool) -> None:
    """Feeds three requests side by side, through slots not in row order, in portions of changing size: long ones (cut into
    pieces that are full, one token over, one short), short ones, single tokens behind them.  ``step(given, live, starts, plan)``
    runs one; ``given`` are the rows as partial sums or as the run's type, in turn.  In bfloat16 runs the rows are bfloat16
    numbers, so even there the result is good to 32-bit."""
    for sizes in ([1000], [128, 60, 2, 40, 1], [257, 3]):
        step.start()
        done, turn = [0] * 3, 0
        while any(d < m for d, m in zip(done, LENGTHS)):
            counts = {i: min(sizes[(turn + i) % len(sizes)], LENGTHS[i] - done[i]) for i in range(3) if done[i] < LENGTHS[i]}
            turn += 1
            live = sorted(counts, key=lambda i: counts[i] == 1)
            long = sum(1 for i in live if counts[i] > 1)
            row = torch.cat([rows[i][done[i]:done[i] + counts[i]] for i in live]).contiguous()
            given = row.to(DEV)
            if turn % 2:  # (halves and quarters of bfloat16 numbers are exact, and so is their sum)
                given = torch.stack([0.5 * row.float(), 0.25 * row.float(), 0.25 * row.float()]).to(DEV)
            starts = [0]
            for i in live:
                starts.append(starts[-1] + counts[i])
            plan = None
            if pieces and long and turn % 3:
                cut, carries = ops.linear_state_pieces([counts[i] for i in live[:long]], ops.decaying_piece)
                plan = (ops.device_ints(cut), ops.device_ints(carries), len(cut), len(carries))
            step(given, live, starts, plan, done)
            for i in live:
                done[i] += counts[i]
        step.finish()


class RetentionStep:
    def __init__(self, ops, dtype, heads, n, p, columns, decay, rows):
        self.ops, self.dtype, self.heads, self.n, self.p, self.columns = ops, dtype, heads, n, p, columns
        self.decay = torch.tensor(decay, dtype=torch.float32, device=DEV)
        x_at, b_at, c_at = columns
        self.want = []
        for row in rows:
            v, k, q = (row.double()[:, at:at + heads * w].view(-1, heads, w) for at, w in ((x_at, p), (b_at, n), (c_at, n)))
            self.want.append(torch.stack([0.25 * plain.retention_walk(q[:, a], k[:, a], v[:, a], float(self.decay[a])) for a in range(heads)], dim=1).flatten(1))

    def start(self):
        self.state = torch.full((6, self.heads, self.p, self.n), float("nan"), device=DEV)
        self.state[SLOTS] = 0.0
        self.got = [torch.zeros_like(w) for w in self.want]

    def __call__(self, given, live, starts, plan, done):
        y, norm = self.ops.decaying_state("fixed", given, self.columns, self.state, ints([SLOTS[i] for i in live]), ints(starts), num_seqs=len(live),
                                          heads=self.heads, groups=self.heads, state_dim=self.n, value_dim=self.p, dtype=self.dtype,
                                          numbers=(self.decay,), scale=0.25, plan=plan)
        assert norm is None
        for j, i in enumerate(live):
            self.got[i][done[i]:done[i] + starts[j + 1] - starts[j]] = y[starts[j]:starts[j + 1]].cpu().double()

    def finish(self):
        for got, want in zip(self.got, self.want):
            near(got, want, torch.float32)
        assert torch.isnan(self.state[[0, 2, 5]]).all()


SIZES = [(4, 24, 16), (1, 1, 7), (3, 33, 70), (6, 64, 64), (2, 128, 48), (4, 136, 8), (2, 256, 72), (2, 300, 20), (8, 48, 40), (1, 512, 33)]
CUT = {(24, 16), (64, 64), (128, 48), (136, 8), (256, 72), (48, 40)}  # (state rows, columns) that bfloat16 runs cut into pieces


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,n,p", SIZES)
def test_a_state_with_a_fixed_decay(ops, dtype, heads, n, p):
    """Decays from ones that forget within a token to ones that never do."""
    g = torch.Generator().manual_seed(heads * 1000 + n)
    columns = (8 * heads * n, 16 * heads * n + 8 * heads * p, 0)  # not side by side, and not in the order x, B, C
    width = columns[1] + 8 * heads * n
    rows = [torch.randn(m, width, generator=g).to(dtype) for m in LENGTHS]
    decay = [(0.999, 0.9, 1.0, 0.01, 0.99, 0.7, 0.9999, 0.5)[a] for a in range(heads)]
    pieces = ops.decaying_pieces_supported(dtype, n, p)
    assert pieces == (dtype == torch.bfloat16 and (n, p) in CUT)
    walked(ops, rows, RetentionStep(ops, dtype, heads, n, p, columns, decay, rows), pieces)


class MemoryStep:
    """The gated rule with its finish behind every step (which moves the running maxima on)."""

    def __init__(self, ops, dtype, heads, n, p, cap, gates, rows):
        self.ops, self.dtype, self.heads, self.n, self.p, self.cap = ops, dtype, heads, n, p, cap
        self.good = 1e-4 if cap < 50.0 else 4e-4  # (the exponents are differences of 32-bit numbers as large as the cap)
        self.first = 2 * heads * n + 2 * heads * p
        self.columns = (2 * heads * n, heads * n, 0)
        self.gate_at = 2 * heads * n + heads * p
        g = torch.Generator().manual_seed(n)
        self.biases = tuple((shift + torch.randn(heads, generator=g)) for shift in gates)
        self.gain = (1.0 + 0.3 * torch.randn(heads * p, generator=g)).to(dtype)
        self.scale = n ** -0.5
        self.want = []
        for row in rows:
            wide = row.double()
            q, k, v, z = (wide[:, at:at + heads * w].view(-1, heads, w) for at, w in
                          ((0, n), (heads * n, n), (2 * heads * n, p), (self.gate_at, p)))
            i, f = plain.capped_gates(wide[:, self.first:self.first + heads] + self.biases[0].double(),
                                      wide[:, self.first + heads:self.first + 2 * heads] + self.biases[1].double(), cap)
            o = torch.stack([plain.memory_walk(q[:, a] * self.scale, k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(heads)], dim=1)
            final = plain.unit_rms(o, 1e-5) * torch.sigmoid(z)
            self.want.append((o, 0.7 * final.flatten(1) * self.gain.double()))

    def start(self):
        self.state = torch.full((6, self.heads, self.p, self.n), float("nan"), device=DEV)
        self.sums = torch.full((6, self.heads, self.n), float("nan"), device=DEV)
        self.tops = torch.full((6, self.heads), float("nan"), device=DEV)
        for held in (self.state, self.sums, self.tops):
            held[SLOTS] = 0.0
        self.got = [(torch.zeros_like(o), torch.zeros_like(y)) for o, y in self.want]

    def __call__(self, given, live, starts, plan, done):
        slots, begin = ints([SLOTS[i] for i in live]), ints(starts)
        y, norm = self.ops.decaying_state(
            "gated", given, self.columns, self.state, slots, begin, num_seqs=len(live), heads=self.heads, groups=self.heads,
            state_dim=self.n, value_dim=self.p, dtype=self.dtype, proj=given, first_gate=self.first,
            numbers=tuple(b.to(DEV) for b in self.biases), cap=self.cap, scale=self.scale, sums=self.sums, tops=self.tops, plan=plan)
        seq_of = ints([j for j in range(len(live)) for _ in range(starts[j + 1] - starts[j])])
        out = self.ops.heads_finish(y, given, self.gate_at, self.heads, 1e-5, self.dtype, gate="sigmoid", gain=self.gain.to(DEV), norm=norm,
                                    tops=self.tops, state_slots=slots, token_seq=seq_of, query_start_loc=begin, scale=0.7).cpu()
        o = y.cpu().double().view(-1, self.heads, self.p)
        norm = norm.cpu().double()
        o = o / (torch.maximum(norm[..., 0].abs(), torch.exp(-norm[..., 1])) + 1e-6)[..., None]
        for j, i in enumerate(live):
            rows = slice(done[i], done[i] + starts[j + 1] - starts[j])
            self.got[i][0][rows] = o[starts[j]:starts[j + 1]]
            self.got[i][1][rows] = out[starts[j]:starts[j + 1]].double()

    def finish(self):
        for (o, y), (want_o, want_y) in zip(self.got, self.want):
            # A head whose n . q is small against its terms, where it is what divides, answers rounding strongly: such tokens
            # (one in fifty, or two) are left out of the comparison of the quotient.
            off = ((o - want_o).abs().amax(dim=-1) / want_o.abs().amax(dim=-1).clamp_min(1e-2 * float(want_o.abs().max()))).flatten().sort().values
            assert float(off[-1 - max(2, len(off) // 50)]) <= self.good, float(off[-1])
            assert torch.isfinite(y).all()
            off = ((y - want_y).abs().amax(dim=-1) / want_y.abs().max()).sort().values
            assert float(off[-1 - max(2, len(off) // 50)]) <= (self.good if self.dtype == torch.float32 else 1e-2), float(off[-1])
        for held in (self.state, self.sums, self.tops):
            assert torch.isnan(held[[0, 2, 5]]).all() and torch.isfinite(held[SLOTS]).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("gates,cap", [((0.0, 3.0), 9.0), ((-4.0, 6.0), 15.0), ((2.0, -1.0), 30.0), ((90.0, 0.0), 120.0), ((-90.0, 9.0), 100.0)])
@pytest.mark.parametrize("heads,n,p", [(4, 24, 16), (3, 33, 70), (6, 64, 64), (2, 256, 72)])
def test_a_memory_with_exponential_gates(ops, dtype, heads, n, p, gates, cap):
    """Gates whose sums are far from 1 in both directions: inputs that weigh e^90 or e^-90, forgetting within a token and
    over hundreds of them.  Nothing overflows, the first tokens' maximum starts at 0."""
    g = torch.Generator().manual_seed(heads * 1000 + n)
    width = 2 * heads * n + 2 * heads * p + 2 * heads
    rows = [torch.randn(m, width + -width % 16, generator=g) for m in LENGTHS]
    for row in rows:
        row[:, width - 2 * heads:width] *= 2.0
    rows = [row.to(dtype) for row in rows]
    pieces = ops.decaying_pieces_supported(dtype, n, p)
    walked(ops, rows, MemoryStep(ops, dtype, heads, n, p, cap, gates, rows), pieces)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,p,tokens,splits", [(1, 5, 3, 0), (3, 24, 70, 2), (4, 256, 9, 11), (2, 1028, 5, 0), (8, 64, 300, 0)])
def test_the_finish_of_heads(ops, dtype, heads, p, tokens, splits):
    """With and without a gain, both gates, a scale, into a buffer of its own and into columns of a wider one."""
    g = torch.Generator().manual_seed(p)
    width, at = heads * p, 4
    y = torch.randn(tokens, width, generator=g)
    proj = torch.randn(max(splits, 1), tokens, at + width + 8, generator=g)
    given = proj.to(DEV) if splits else proj[0].to(dtype).to(DEV)
    z = (proj.sum(0) if splits else proj[0].to(dtype).float())[:, at:at + width]
    gain = (1.0 + 0.3 * torch.randn(width, generator=g)).to(dtype)
    unit = plain.unit_rms(y.view(tokens, heads, p), 1e-3).flatten(1)
    for gate, act in (("silu", plain.silu), ("sigmoid", torch.sigmoid)):
        near(ops.heads_finish(y.to(DEV), given, at, heads, 1e-3, dtype, gate=gate), unit * act(z), dtype)
        buffer = torch.full((tokens, width + 24), 3.0, dtype=dtype, device=DEV)
        out = ops.heads_finish(y.to(DEV), given, at, heads, 1e-3, dtype, gate=gate, gain=gain.to(DEV), scale=-0.6, out=(buffer, 16))
        assert out.data_ptr() == buffer.data_ptr()
        near(buffer[:, 16:16 + width], -0.6 * unit * act(z) * gain.float(), dtype)
        assert bool((buffer[:, :16] == 3).all()) and bool((buffer[:, 16 + width:] == 3).all())


# ---------------------------------------------------------------------------------------------
# mechanisms alone: what the other parts learned
# ---------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hidden,tokens", [(51, 5), (64, 70), (2048, 70), (4096, 2), (5001, 2)])
def test_the_layer_norm_without_a_bias(ops, dtype, hidden, tokens):
    g = torch.Generator().manual_seed(hidden)
    residual, pending = 3.0 + torch.randn(tokens, hidden, generator=g), 5.0 + torch.randn(3, tokens, hidden, generator=g)
    post, own = ((1 + 0.3 * torch.randn(hidden, generator=g)).to(dtype) for _ in range(2))
    for with_post in (False, True):
        p = pending.sum(0)
        total = residual + (0.7 * plain.centred_norm(p, post.float(), 1e-5) if with_post else p)
        stream = residual.clone().to(DEV)
        got = ops.add_layer_norm(stream, pending.to(DEV), dtype, norm=(own.to(DEV), None, 1e-4),
                                 pending_norm=(post.to(DEV), None, 1e-5, 0.7) if with_post else None)
        near(got, plain.centred_norm(total, own.float(), 1e-4), dtype)
        near(stream, total, torch.float32)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_scaled_embedding_and_logits(ops, dtype):
    g = torch.Generator().manual_seed(2)
    table = torch.randn(30, 51, generator=g).to(dtype)
    ids = ints([3, 0, 29, 3])
    near(ops.embed(table.to(DEV), ids, scale=3.0), 3.0 * table[ids.cpu().long()].float(), torch.float32)
    x = 20 * torch.randn(3, 700, generator=g)
    near(ops.scale_cap(x.clone().to(DEV), scale=0.25), 0.25 * x, torch.float32)
    near(ops.scale_cap(x.clone().to(DEV), scale=-2.0, cap=5.0), 5.0 * torch.tanh(-2.0 * x / 5.0), torch.float32)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,ff", [(40, 28), (51, 20), (64, 96), (2048, 512)])
@pytest.mark.parametrize("tokens", [1, 5, 30, 100, 200, 700])
def test_the_gated_unit_with_biases(ops, dtype, width, ff, tokens):
    """Every product that can run it: few rows, many, the library's, an inner size 16-byte accesses do not divide."""
    from turboserve_amd.kernels.ops import GELU_TANH_RULE

    g = torch.Generator().manual_seed(width + tokens)
    x = torch.randn(tokens, width, generator=g).to(dtype)
    t = {"f.gate": width ** -0.5 * torch.randn(ff, width, generator=g), "f.up": width ** -0.5 * torch.randn(ff, width, generator=g),
         "f.gate.b": 0.7 * torch.randn(ff, generator=g), "f.up.b": 0.7 * torch.randn(ff, generator=g)}
    t = {name: v.to(dtype) for name, v in t.items()}
    wide = {name: v.float() for name, v in t.items()}
    want = plain.gelu_tanh(plain.projected("f.gate", wide, x.float())) * plain.projected("f.up", wide, x.float())
    weight = torch.stack([t["f.gate"], t["f.up"]], dim=1).reshape(2 * ff, width).contiguous().to(DEV)
    bias = torch.stack([t["f.gate.b"], t["f.up.b"]], dim=1).reshape(-1).contiguous().to(DEV)
    near(ops.linear_swiglu(x.to(DEV), weight, GELU_TANH_RULE, bias), want, dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top", [(5, 2), (3, 3), (70, 4), (8, 1)])
def test_the_router_with_a_bias(ops, dtype, experts, top):
    g = torch.Generator().manual_seed(experts)
    x, router = torch.randn(40, 64, generator=g).to(dtype), (0.5 * torch.randn(experts, 64, generator=g)).to(dtype)
    bias = 3.0 * torch.randn(experts, generator=g)
    taken, weights, gate = ops.moe_route(x.to(DEV), router.to(DEV), top=top, groups=1, keep=1, scale=1.0, softmax=True, bias=bias.to(DEV))
    assert gate is None
    z = x.float() @ router.float().T + bias
    for t in range(40):
        want = plain.chosen(z[t], top)
        assert taken[t].tolist() == [e for e, _ in want]
        near(weights[t], torch.stack([w for _, w in want]), torch.float32)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("normed", [False, True])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,turned,tokens", [
    (4, 2, 16, 24, 16, 40), (3, 3, 12, 12, 8, 45), (2, 1, 128, 128, 128, 70), (8, 1, 128, 64, 64, 35), (1, 1, 64, 80, 48, 33), (6, 2, 72, 40, 32, 90),
    (2, 2, 40, 40, 12, 37), (3, 1, 96, 96, 96, 5)])
def test_the_store_turns_halves_of_a_heads_first_elements(ops, dtype, normed, heads, kv_heads, dim, vdim, turned, tokens):
    """In prompts (also where a pair lies in two lanes) and in steps of few tokens, with a norm per head and without."""
    g = torch.Generator().manual_seed(dim + tokens)
    page, first = 8, 29
    proj = torch.randn(tokens, (heads + kv_heads) * dim + kv_heads * vdim, generator=g).to(dtype)
    gains = [(1 + 0.3 * torch.randn(dim, generator=g)).to(dtype) for _ in range(2)]
    rot = {"base": 70.0, "dims": turned}
    angles = torch.outer(torch.arange(first + tokens, dtype=torch.float64), 70.0 ** (-2.0 * torch.arange(turned // 2, dtype=torch.float64) / turned))
    padded = torch.cat([torch.zeros(first, proj.shape[1]), proj.float()])

    def turn(columns, count, gain):
        x = padded[:, columns:columns + count * dim].view(-1, count, dim)
        return plain.turn_halves(plain.unit_rms(x, 1e-5) * gain.float() if normed else x, rot)[first:]

    pages = -(-(first + tokens) // page)
    order = torch.randperm(pages, generator=g)
    slots = torch.tensor([int(order[p // page]) * page + p % page for p in range(first, first + tokens)])
    k_pages = torch.zeros(pages, kv_heads, page, dim, dtype=dtype, device=DEV)
    v_pages = torch.zeros(pages, kv_heads, vdim, page, dtype=dtype, device=DEV)
    q, stride = ops.head_norm_store(
        proj.clone().to(DEV), k_pages, v_pages, *(gain.to(DEV) if normed else None for gain in gains), 1e-5, ints(range(first, first + tokens)),
        slots.to(torch.int32).to(DEV), heads, kv_heads, dim, vdim, page, dtype, cos=angles.cos().float().to(DEV),
        sin=angles.sin().float().to(DEV), max_position=first + tokens - 1)
    near(q.view(tokens, -1)[:, :heads * dim], turn(0, heads, gains[0]).reshape(tokens, -1), dtype)
    near(k_pages[slots // page, :, slots % page], turn(heads * dim, kv_heads, gains[1]), dtype)
    near(v_pages[slots // page, :, :, slots % page], proj.float()[:, (heads + kv_heads) * dim:].view(tokens, kv_heads, vdim), dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 16, 24), (3, 1, 20, 12), (8, 1, 64, 80)])
def test_attention_scales_and_places_its_heads(ops, dtype, heads, kv_heads, dim, vdim):
    """A portion and a single token behind it, the keys of the single token shared out over several workgroups: the same
    numbers as without a place, times the scale, in the columns asked for and nowhere else."""
    g = torch.Generator().manual_seed(dim)
    page, pages, lens, contexts = 16, 40, [70, 1], [90, 400]
    k = torch.randn(pages, kv_heads, page, dim, generator=g).to(dtype).to(DEV)
    v = torch.randn(pages, kv_heads, vdim, page, generator=g).to(dtype).to(DEV)
    table = torch.randperm(pages, generator=g)[:32].to(torch.int32).view(1, 32).repeat(2, 1).contiguous().to(DEV)
    q = torch.randn(71, heads * dim, generator=g).to(dtype).to(DEV)
    positions = ints([*range(20, 90), 399])
    seqs, width = ints([0] * 70 + [1]), heads * vdim
    calls = [lambda **more: ops.paged_attention_generic(q, heads * dim, k, v, table, seqs, positions, heads, 0.3, None, chunk=333, **more)]
    if ops.tiled_attention_supported(dtype, dim, vdim, page, heads * dim):
        tiles = ops.device_ints(ops.attention_tile_list(lens[:1], contexts[:1], chunk=333))
        calls.append(lambda **more: ops.attention_tiles(
            q, heads * dim, k, v, table, ints([0, 70, 71]), ints(contexts), tokens=71, heads=heads, scale=0.3, prefill_tiles=tiles,
            num_prefill_seqs=1, num_decode_seqs=1, max_decode_context=400, chunk=333, **more))
    for call in calls:
        bare = call().float().cpu()
        buffer = torch.full((71, width + 40), 3.0, dtype=dtype, device=DEV)
        call(out_scale=-0.6, out=(buffer, 8))
        near(buffer[:, 8:8 + width], -0.6 * bare, dtype)
        assert bool((buffer[:, :8] == 3).all()) and bool((buffer[:, 8 + width:] == 3).all())


# ---------------------------------------------------------------------------------------------
# mechanisms alone: models of one layer
# ---------------------------------------------------------------------------------------------

QUIET = nt.retention(1, 8, 8, 0.9)
ALONE = {
    "memory": [nt.layer(nt.memory(4, 16, 24, 9.0))],
    "memory_one_head": [nt.layer(nt.memory(1, 12, 9, 6.0))],
    "memory_one_row": [nt.layer(nt.memory(3, 1, 8, 12.0))],
    "memory_wide": [nt.layer(nt.memory(2, 136, 72, 15.0))],
    "memory_small_cap": [nt.layer(nt.memory(2, 16, 16, 0.5))],
    "memory_run_twice": [nt.layer(nt.memory(2, 16, 8, 9.0)), nt.again([nt.layer(nt.memory(2, 16, 8, 9.0))], 0)],
    "chunks": [nt.layer(nt.parallel(nt.attention(4, 2, 16, chunk=20, rot=16, base=100.0), QUIET, 1.0, 0.0))],
    "chunks_of_one": [nt.layer(nt.parallel(nt.attention(2, 1, 16, 8, chunk=1, rot=4), QUIET, 1.0, 0.1))],
    "chunks_no_rotation": [nt.layer(nt.parallel(nt.attention(3, 3, 12, 20, chunk=9, scale=0.6), QUIET, 1.0, 0.0))],
    "chunks_matrix_cores": [nt.layer(nt.parallel(nt.attention(8, 1, 64, 80, chunk=48, rot=24, base=300.0), QUIET, 0.8, 0.3))],
    "no_chunks": [nt.layer(nt.parallel(nt.attention(4, 2, 32, rot=32), QUIET, 1.0, 0.2))],
    "no_chunks_other_values": [nt.layer(nt.parallel(nt.attention(4, 2, 32, 16, rot=8), QUIET, 1.0, 0.2))],
    "retention": [nt.layer(nt.parallel(nt.attention(1, 1, 8, chunk=4), nt.retention(3, 16, 24, 0.9, 0.99, 1.0), 0.0, 1.0))],
    "retention_wide": [nt.layer(nt.parallel(nt.attention(1, 1, 8, chunk=4), nt.retention(2, 136, 72, 0.95, 0.999), 0.2, 1.0))],
    "retention_odd": [nt.layer(nt.parallel(nt.attention(1, 1, 8, chunk=4), nt.retention(2, 7, 9, 0.3, 0.97), -0.5, 1.3))],
    "pair_run_twice": [nt.layer(nt.parallel(nt.attention(2, 1, 16, 8, chunk=10, rot=8), nt.retention(2, 8, 16, 0.9, 0.99), 0.7, 0.6)),
                       nt.again([nt.layer(nt.parallel(nt.attention(2, 1, 16, 8, chunk=10, rot=8), nt.retention(2, 8, 16, 0.9, 0.99), 0.7, 0.6))], 0)],
    "dense": [nt.layer(nt.memory(1, 8, 8, 5.0), nt.dense(52))],
    "experts": [nt.layer(nt.memory(1, 8, 8, 5.0), nt.moe(7, 3, 28))],
    "experts_shared": [nt.layer(nt.memory(1, 8, 8, 5.0), nt.moe(4, 1, 32, 20))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", sorted(ALONE))
def test_one_layer_models(tmp_path, which, dtype):
    """Whole, token by token from the start, and in portions, against the plain implementation."""
    folder = nt.make_model_dir(tmp_path / "m", nt.model(ALONE[which]), 31, stored_as(dtype), std=0.2)
    requests = {"a": tokens_of(61, 140, 1), "b": tokens_of(61, 3, 2)}
    want = {rid: expect(folder, tokens, dtype) for rid, tokens in requests.items()}
    for steps in (th.whole(requests), th.prefix_then_single(requests, tail=139), th.portions(requests, (2, 5, 71, 3))):
        got = th.collect(steps, run_trace(folder, dtype, 8, steps), requests)
        for rid in requests:
            assert excess(got[rid], want[rid], dtype) <= 1.0, (which, rid)


# ---------------------------------------------------------------------------------------------
# whole models, every cutting
# ---------------------------------------------------------------------------------------------


@pytest.fixture(scope="module", params=sorted(nt.TINY))
def case(request, tmp_path_factory):
    config, seed, page = nt.TINY[request.param]
    base = tmp_path_factory.mktemp(f"ninenex_{request.param}")
    folders = {dtype: nt.make_model_dir(base / dtype, config, seed, stored_as(dtype)) for dtype in ("float32", "bfloat16")}
    lengths = (1, 2, 37, 180, 70, 9)
    requests = {f"r{i}": tokens_of(config["vocab"], n, 100 * seed + i) for i, n in enumerate(lengths)}
    expected = {dtype: {rid: expect(folder, tokens, dtype) for rid, tokens in requests.items()} for dtype, folder in folders.items()}
    return {"name": request.param, "page": page, "folders": folders, "requests": requests, "expected": expected}


def check_against_plain(case, dtype: str, steps: list[dict], **more) -> None:
    outputs = run_trace(case["folders"][dtype], dtype, case["page"], steps, **more)
    got = th.collect(steps, outputs, case["requests"])
    for rid, want in case["expected"][dtype].items():
        worst = excess(got[rid], want, dtype)
        assert worst <= 1.0, f"{case['name']} {dtype} {rid}: {worst:.2f} times the bound"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompts(case, dtype):
    check_against_plain(case, dtype, th.whole(case["requests"]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_prefix_then_token_by_token(case, dtype):
    check_against_plain(case, dtype, th.prefix_then_single(case["requests"], tail=40))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(2, 3, 5, 2, 16, 7), (33, 2, 70, 64), (1, 2)])
def test_portions_of_changing_size(case, dtype, sizes):
    check_against_plain(case, dtype, th.portions(case["requests"], sizes))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_on_pages_and_slots_that_are_used_again(case, dtype):
    """Three requests live at a time out of six, on a pool sized for the peak and three state slots: every
    page and slot serves several requests, and what one left there must not reach the next."""
    steps = th.mixed(case["requests"], (7, 2, 19, 66, 3), max_live=3, decode_tail=9)
    check_against_plain(case, dtype, steps, max_live=3)


def test_long_decoding(case):
    """One short prompt, then 180 tokens one by one (recorded steps), in 32-bit: states, sums and maxima are carried
    through every one of them, chunk after chunk."""
    config = nt.TINY[case["name"]][0]
    tokens = tokens_of(config["vocab"], 186, 4242)
    requests = {"long": tokens}
    steps = th.prefix_then_single(requests, tail=180)
    got = th.collect(steps, run_trace(case["folders"]["float32"], "float32", case["page"], steps), requests)["long"]
    assert excess(got, expect(case["folders"]["float32"], tokens, "float32"), "float32") <= 1.0, case["name"]


def test_cuttings_agree_in_32_bit(case):
    """The logits of a position do not depend on how its request was cut or batched, beyond rounding."""
    folder, page = case["folders"]["float32"], case["page"]
    ways = {"whole": th.whole(case["requests"]), "single": th.prefix_then_single(case["requests"], tail=40),
            "portions": th.portions(case["requests"], (2, 5, 3, 24)), "mixed": th.mixed(case["requests"], (5, 2, 21, 80), max_live=4)}
    results = {name: th.collect(steps, run_trace(folder, "float32", page, steps), case["requests"]) for name, steps in ways.items()}
    for name, got in results.items():
        for rid, base in results["whole"].items():
            scale = base.abs().amax(dim=-1, keepdim=True).clamp_min(1.0)
            assert float(((got[rid] - base).abs() / scale).max()) <= 5e-5, (name, rid)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_replay_program(case, dtype, tmp_path):
    """``bin/trace_run`` itself on a model folder of this design, steps that want nothing included."""
    if case["name"] != "A":
        pytest.skip("one configuration is enough for the subprocess test")
    steps = th.mixed(case["requests"], (7, 2, 19, 66, 3), max_live=3, decode_tail=9)
    for record in steps[1::3]:
        for entry in record["entries"]:
            entry["want"] = []
    out = tmp_path / "out"
    proc = subprocess.run(
        [sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(case["folders"][dtype]), "--dtype", dtype,
         "--out", str(out), "--max-tokens", str(th.peak_tokens(steps)), "--page-size", str(case["page"])],
        input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600,
    )
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [line for line in proc.stdout.splitlines() if line.startswith("done ")] == [f"done {s['step']}" for s in steps]
    import numpy as np

    vocab = nt.TINY["A"][0]["vocab"]
    position = {rid: 0 for rid in case["requests"]}
    got, want, bound = [], [], []
    for record in steps:
        wanted = sum(len(e["want"]) for e in record["entries"])
        path = out / f"{record['step']}.f32"
        assert path.exists() == bool(wanted)
        if wanted:
            got.append(torch.from_numpy(np.fromfile(path, dtype="<f4").reshape(wanted, vocab).copy()))
        for entry in record["entries"]:
            for place in entry["want"]:
                row, limit = (t[position[entry["id"]] + place] for t in case["expected"][dtype][entry["id"]])
                want.append(row)
                bound.append(limit)
            position[entry["id"]] += len(entry["tokens"])
    assert excess(torch.cat(got), (torch.stack(want), torch.stack(bound)), dtype) <= 1.0


def random_config(rng: random.Random) -> dict:
    layers: list[dict] = []
    for index in range(rng.randint(1, 6)):
        if layers and rng.random() < 0.3:
            source = rng.randrange(len(layers))
            layers.append({**layers[source], "weights_of": source})
            continue
        mlp = rng.choice([None, nt.dense(rng.choice([12, 44, 64])), nt.moe(rng.choice([2, 5, 9]), rng.choice([1, 2]), rng.choice([12, 32]),
                                                                         rng.choice([None, 20, 48]))])
        if rng.random() < 0.5:
            layers.append(nt.layer(nt.memory(rng.choice([1, 2, 3, 6]), rng.choice([3, 8, 16, 20, 64, 96]), rng.choice([4, 8, 20, 40, 64]),
                                             rng.choice([0.7, 4.0, 10.0, 25.0])), mlp))
            continue
        kv, dim = rng.choice([1, 1, 2, 3]), rng.choice([8, 12, 16, 20, 32, 64])
        left = nt.attention(kv * rng.choice([1, 2, 3, 4]), kv, dim, rng.choice([dim, dim, 8, 24, 40]), chunk=rng.choice([None, 1, 5, 16, 50, 64, 500]),
                            scale=rng.choice([None, 0.2, 0.5]), rot=rng.choice([None, 2, dim // 2, dim]), base=rng.choice([10.0, 1000.0, 1e6]))
        heads = rng.choice([1, 2, 3])
        right = nt.retention(heads, rng.choice([4, 8, 24, 64]), rng.choice([6, 8, 32, 64]), *(rng.choice([0.2, 0.9, 0.99, 0.9990234375, 1.0]) for _ in range(heads)))
        layers.append(nt.layer(nt.parallel(left, right, rng.choice([1.0, 0.6, -0.5]), rng.choice([1.0, 0.4, 1.7])), mlp))
    return nt.model(layers, vocab=rng.choice([50, 97, 256]), width=rng.choice([40, 51, 64, 72, 96, 100, 128]), eps=rng.choice([1e-6, 1e-5]),
                    embedding=rng.choice([0.5, 1.0, 4.0]), logits=rng.choice([0.3, 1.0, 2.5]))


@pytest.mark.parametrize("trial", range(8))
def test_random_configurations_replay_like_plain(trial, tmp_path):
    """Seeded random configurations: one to six layers of either mixer in any order, layers that run with any earlier
    one's tensors, chunks from one token to longer than the prompt or none, rotation of two elements, half a head, a whole
    head or none, every kind of feed-forward; whole, token by token and mixed."""
    rng = random.Random(9000 + trial)
    config = random_config(rng)
    lengths = [rng.randint(1, 6), rng.randint(10, 60), rng.randint(100, 160), rng.randint(20, 90)]
    requests = {f"r{i}": [rng.randrange(config["vocab"]) for _ in range(n)] for i, n in enumerate(lengths)}
    for dtype in ("float32", "bfloat16"):
        folder = nt.make_model_dir(tmp_path / dtype, config, trial, stored_as(dtype))
        want = {rid: expect(folder, tokens, dtype) for rid, tokens in requests.items()}
        ways = (th.whole(requests), th.prefix_then_single(requests, tail=20),
                th.mixed(requests, (7, 2, 40, 150, 3), max_live=4, decode_tail=5))
        for steps in ways:
            outputs = run_trace(folder, dtype, 16, steps, max_tokens=th.peak_tokens(steps))
            got = th.collect(steps, outputs, requests)
            together = (torch.cat([want[rid][0] for rid in requests]), torch.cat([want[rid][1] for rid in requests]))
            assert excess(torch.cat([got[rid] for rid in requests]), together, dtype) <= 1.0, (trial, dtype, config)


# ---------------------------------------------------------------------------------------------
# one key that a query rests on: just inside and just outside its chunk, at page borders, at the first positions
# ---------------------------------------------------------------------------------------------

MARK, ASKS, OTHER = 7, 9, 11  # the token that is looked for, the token whose query looks for it, one that is neither


def marked_model(folder, dtype: torch.dtype, chunk: int | None):
    """One pair whose query of ``ASKS`` and key of ``MARK`` point the same way in the part of a head that is not turned, with
    a scale under which that one score stands above all others, and a value of ``MARK`` that reaches the logits.  No other
    token has anything in the two channels that make them; the retention beside it is switched off."""
    config = nt.model([nt.layer(nt.parallel(nt.attention(2, 1, 16, 24, chunk=chunk, scale=1.5, rot=8, base=100.0), QUIET, 1.0, 0.5))],
                      vocab=40, width=32)
    tensors = nt.draw_tensors(config, 5, torch.float32, 0.1)
    tensors["embed"][:, :2] = 0.0
    tensors["embed"][MARK, 0] = 3.0
    tensors["embed"][ASKS, 1] = 3.0
    tensors["l0.norm1"][:] = 1.0
    towards = torch.zeros(16)
    towards[8:] = torch.tensor([1.0, -1.0, 1.0, 1.0, -1.0, 1.0, -1.0, -1.0])
    tensors["l0.mix.right.o"][:] = 0.0
    tensors["l0.mix.left.k"][:, 0], tensors["l0.mix.left.k"][:, 1] = 6.0 * towards, 0.0
    tensors["l0.mix.left.v"][:, 0] = 4.0 * torch.randn(24, generator=torch.Generator().manual_seed(3))
    for head in range(2):
        tensors["l0.mix.left.q"][16 * head:16 * head + 16, 1] = 6.0 * towards
        tensors["l0.mix.left.q"][16 * head:16 * head + 16, 0] = 0.0
    tensors = {name: t.to(dtype).contiguous() for name, t in tensors.items()}
    return nt.make_model_dir(folder, config, 0, tensors=tensors)


def moved(raw: dict, tensors: dict, tokens: list[int], place: int) -> float:
    """How far the plain implementation's logits at ``place`` move when the mark goes, relative to the largest."""
    have = plain.forward(raw, tensors, tokens)[place]
    without = plain.forward(raw, tensors, [t if t != MARK else OTHER for t in tokens])[place]
    return float((have - without).abs().max() / have.abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk,asks_at,mark_at", [
    (20, 39, 20), (20, 39, 19), (20, 40, 40 - 20), (20, 40, 39), (20, 119, 100), (20, 119, 99), (20, 19, 0), (20, 20, 0), (20, 5, 1),
    (64, 127, 64), (64, 127, 63), (64, 128, 127), (64, 130, 128), (64, 63, 0), (7, 48, 42), (7, 48, 41), (48, 95, 48), (48, 95, 47),
    (None, 130, 0), (None, 130, 1), (None, 130, 16), (None, 130, 127),
])
def test_a_key_inside_a_chunk_is_found_and_one_outside_is_not(tmp_path, dtype, chunk, asks_at, mark_at):
    """The plain implementation says what the mark is worth: much inside the chunk, nothing outside, where a chunk one token
    longer (planted in the plain implementation) would see it.  The engine agrees in every cutting: whole, the last tokens
    one by one, portions that end inside chunks and pages."""
    folder = marked_model(tmp_path / "m", stored_as(dtype), chunk)
    g = torch.Generator().manual_seed(mark_at)
    tokens = [t if t not in (MARK, ASKS) else OTHER for t in torch.randint(0, 40, (asks_at + 3,), generator=g).tolist()]
    tokens[asks_at], tokens[mark_at] = ASKS, MARK
    raw, tensors = nt.read_model_dir(folder)
    inside = chunk is None or asks_at // chunk == mark_at // chunk
    worth = moved(raw, tensors, tokens, asks_at)
    assert worth > 0.2 if inside else worth < 1e-5, worth
    if not inside:
        open_end = json.loads(json.dumps(raw))
        open_end["layers"][0]["mixer"]["left"].pop("mask")
        assert moved(open_end, tensors, tokens, asks_at) > 0.2
    want, bound = expect(folder, tokens, dtype)
    requests = {"m": tokens}
    for steps in (th.whole(requests), th.prefix_then_single(requests, tail=min(12, asks_at + 2)), th.portions(requests, (max(1, asks_at), 1, 2)),
                  th.portions(requests, (5, 2, 16, 3))):
        got = th.collect(steps, run_trace(folder, dtype, 16, steps), requests)["m"]
        assert excess(got[asks_at:], (want[asks_at:], bound[asks_at:]), "float32") <= 1.0


# ---------------------------------------------------------------------------------------------
# state that has to last, and where it starts
# ---------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["memory", "retention"])
def test_what_a_token_left_in_the_state_hundreds_of_tokens_back_still_counts(tmp_path, dtype, which):
    """Layers that hardly forget: a token 230 positions back changes the last logits, and the engine follows it whole, token
    by token and in portions."""
    if which == "memory":
        layers = [nt.layer(nt.memory(4, 16, 16, 9.0))]
    else:
        layers = [nt.layer(nt.parallel(nt.attention(1, 1, 8, chunk=4), nt.retention(2, 16, 16, 1.0, 0.9990234375), 0.1, 1.0))]
    config = nt.model(layers, vocab=40, width=32)
    tensors = nt.draw_tensors(config, 8, torch.float32, 0.25)
    channel = tensors["embed"][:, 3]
    channel[:] = 0.0
    tensors["embed"][MARK, 3] = 9.0  # a channel of its own, which keys and values read strongly
    for name in ("l0.mix.k", "l0.mix.v", "l0.mix.right.k", "l0.mix.right.v"):
        if name in tensors:
            tensors[name][:, 3] *= 6.0
    if which == "memory":
        tensors["l0.mix.f.b"][:] = 8.0
        tensors["l0.mix.f"] *= 0.1
        tensors["l0.mix.i"] *= 0.1
        tensors["l0.mix.i"][:, 3] = 1.0  # its input gate opens wide
    tensors = {name: t.to(stored_as(dtype)).contiguous() for name, t in tensors.items()}
    folder = nt.make_model_dir(tmp_path / "m", config, 0, tensors=tensors)
    raw, loaded = nt.read_model_dir(folder)
    tokens = [t if t != MARK else OTHER for t in tokens_of(40, 240, 77)]
    tokens[9] = MARK
    assert moved(raw, loaded, tokens, 239) > 0.05
    want = expect(folder, tokens, dtype)
    requests = {"m": tokens}
    for steps in (th.whole(requests), th.prefix_then_single(requests, tail=200), th.portions(requests, (9, 2, 64, 1, 130))):
        got = th.collect(steps, run_trace(folder, dtype, 16, steps), requests)["m"]
        assert excess(got, want, dtype) <= 1.0


def test_a_read_out_is_divided_by_one_at_least(tmp_path, monkeypatch):
    """Input gates so low that a memory holds next to nothing: its heads are then small against the norm's eps.  Divided by
    the sum of keys alone (planted in the plain implementation) they would be large, and the engine's are not."""
    config = nt.model([nt.layer(nt.memory(2, 8, 8, 20.0))], vocab=40, width=32, eps=1e-3)
    tensors = nt.draw_tensors(config, 3, torch.float32, 0.25)
    tensors["l0.mix.i.b"][:] = -6.0
    folder = nt.make_model_dir(tmp_path / "m", config, 0, tensors=tensors)
    raw, loaded = nt.read_model_dir(folder)
    tokens = tokens_of(40, 40, 5)
    want, bound = expect(folder, tokens, "float32")
    monkeypatch.setattr(plain, "least", torch.zeros_like)
    other = plain.forward(raw, loaded, tokens).double()
    monkeypatch.undo()
    assert float(((other - want).abs().amax(dim=-1) / bound).median()) > 20.0
    for steps in (th.whole({"m": tokens}), th.prefix_then_single({"m": tokens}, tail=39)):
        got = th.collect(steps, run_trace(folder, "float32", 16, steps), {"m": tokens})["m"]
        assert excess(got, (want, bound), "float32") <= 1.0


# ---------------------------------------------------------------------------------------------
# generation through the engine's own entry point and the command line
# ---------------------------------------------------------------------------------------------


@pytest.mark.parametrize("name,blocks", [("A", 40), ("B", 40), ("C", 40), ("A", 10)])
def test_greedy_generation_through_the_engine(tmp_path, name, blocks):
    """Twice on one engine, steps launched ahead (the token before the one that is fed is then known on the device
    only); with few pages requests are preempted and run again from their first token."""
    from turboserve_amd.config.engine_config import EngineConfig, SchedulerConfig
    from turboserve_amd.engine.llm_engine import LLMEngine
    from turboserve_amd.sampling.params import SamplingParams

    config, seed, page = nt.TINY[name]
    folder = nt.make_model_dir(tmp_path / "gen", config, seed + 5, torch.float32, std=0.2)
    raw, tensors = nt.read_model_dir(folder)
    prompts = [tokens_of(config["vocab"], n, 900 + n) for n in (3, 21, 1, 50)]
    new = 30
    want = [nt.greedy(raw, tensors, prompt, new) for prompt in prompts]
    engine = LLMEngine(EngineConfig(
        model=str(folder), dtype="float32",
        scheduler=SchedulerConfig(max_num_seqs=4, max_num_batched_tokens=64, block_size=page, num_blocks=blocks),
    ))
    outputs = engine.generate(prompts, SamplingParams(max_tokens=new, temperature=0.0, ignore_eos=True))
    assert [out.new_token_ids for out in outputs] == want
    again = engine.generate(list(reversed(prompts)), SamplingParams(max_tokens=new, temperature=0.0, ignore_eos=True))
    assert [out.new_token_ids for out in again] == list(reversed(want))


def test_a_model_of_memories_alone_is_served_without_pages(tmp_path):
    """No layer keeps keys: the engine has state slots and no page pool, and requests end by their length."""
    from turboserve_amd.config.engine_config import EngineConfig, SchedulerConfig
    from turboserve_amd.engine.llm_engine import LLMEngine
    from turboserve_amd.sampling.params import SamplingParams

    layers = [nt.layer(nt.memory(4, 16, 24, 9.0), nt.dense(36)), nt.layer(nt.memory(2, 32, 16, 12.0))]
    folder = nt.make_model_dir(tmp_path / "m", nt.model([*layers, nt.again(layers, 0)]), 3, torch.float32, std=0.2)
    raw, tensors = nt.read_model_dir(folder)
    prompts = [tokens_of(61, n, n) for n in (5, 70, 1)]
    engine = LLMEngine(EngineConfig(model=str(folder), dtype="float32", scheduler=SchedulerConfig(
        max_num_seqs=2, max_num_batched_tokens=32, block_size=16, num_blocks=None)))
    outputs = engine.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert [out.new_token_ids for out in outputs] == [nt.greedy(raw, tensors, prompt, 12) for prompt in prompts]


def test_the_command_line_serves_the_design(tmp_path, capsys):
    """``engine random-model`` writes a folder from a config.json of the design, ``engine generate``
    completes prompts given as token ids with the plain implementation's greedy tokens, and ``engine
    kv-size`` sizes its cache."""
    import re

    from turboserve_amd import cli

    config, _, page = nt.TINY["A"]
    source = tmp_path / "config.json"
    source.write_text(json.dumps(config))
    folder = tmp_path / "model"
    assert cli.main(["engine", "random-model", "--config", str(source), "--out", str(folder), "--seed", "4", "--dtype", "float32"]) == 0
    raw, tensors = nt.read_model_dir(folder)
    prompts = [tokens_of(config["vocab"], n, 600 + n) for n in (4, 19)]
    capsys.readouterr()
    args = ["engine", "generate", "--model", str(folder), "--dtype", "float32", "--max-tokens", "12", "--ignore-eos",
            "--num-blocks", "24", "--block-size", str(page)]
    assert cli.main(args + [a for p in prompts for a in ("--prompt-ids", ",".join(map(str, p)))]) == 0
    shown = [json.loads(m) for m in re.findall(r"^output \d+: (\[.*\])$", capsys.readouterr().out, flags=re.M)]
    assert len(shown) == len(prompts)
    for prompt, got in zip(prompts, shown):
        tokens = list(prompt)
        for token in got:  # the written model's weights are small: equal logits are allowed for
            logits = plain.forward(raw, tensors, tokens)[-1]
            assert float(logits.max() - logits[token]) <= 1e-4 * float(logits.abs().max().clamp_min(1.0))
            tokens.append(token)
    assert cli.main(["engine", "kv-size", "--model", str(folder), "--dtype", "bfloat16", "--max-model-len", "64",
                     "--block-size", str(page)]) == 0
    sizing = capsys.readouterr().out
    sizing = json.loads(sizing[sizing.index("{"):])
    assert sorted(sizing["bytes_per_block"]) == sorted([2 * 2 * (16 + 24) * 2 * page, (8 + 8) * 2 * page]) and sizing["activation_bytes"] > 0
