"""Gozatar through the step function, the cache manager, the scheduler and the entry point, against the plain
implementation, under every way of cutting the work; and each of its mechanisms' kernels alone.

The model-level runs in float32 use folders whose routers choose freely; those in bfloat16 use the same folders with
steady routers (``cases.steady`` says why). The routers' free choice is covered where it can be pinned: the choice
kernel on given logits, and the experts' kernels on given choices."""

import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import helpers
from tests import gozatar_cases as cases
from tests.helpers import Request
from tests.packed import CUTS, PackedStep
from tests.plain import gozatar_plain as plain

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [torch.float32, torch.bfloat16]
DTYPE_IDS = ["fp32", "bf16"]
NAMES = ["P", "Q", "R", "S"]
DEV = "cuda:0"
F64 = torch.float64


def _runner(folder, dtype, n_pages=64, max_requests=4, graphs=False):
    from kestrel_amd.engine.loading import load_model, make_runner

    net = load_model(folder, dtype, torch.device(DEV))
    runner = make_runner(net, 16, n_pages, max_requests, enable_graphs=graphs)
    helpers.poison_cache(runner)
    return runner


def _ids(folder, seed, count):
    return helpers.random_ids(seed, count, cases.config_of(folder)["vocab"])


_EXPECTED = {}


def _expected(folder, ids):
    key = (folder, tuple(ids))
    if key not in _EXPECTED:
        _EXPECTED[key] = plain.forward(cases.config_of(folder), cases.stored_weights(folder), ids)
    return _EXPECTED[key]


_NOISY = {}


def _what_rounding_does(folder, ids):
    """Per row of logits, how far the plain implementation itself moves (as a share of the row's spread) when every weight is
    off by a relative 2 ** -8, about what rounding to bfloat16 does to every intermediate value. The design amplifies that
    without any fault where little has been summed up yet: at a sequence's first tokens a head of the recurrence reads one
    or two products ``q . k``, which may nearly cancel, and every head is divided by its own root mean square."""
    if folder not in _NOISY:
        gen = torch.Generator().manual_seed(99)
        _NOISY[folder] = [{k: (v.double() * (1 + 2.0 ** -8 * torch.randn(v.shape, generator=gen, dtype=F64)))
                           for k, v in cases.stored_weights(folder).items()} for _ in range(3)]
    want = _expected(folder, ids)
    worst = torch.zeros(want.shape[0], dtype=F64)
    for noisy in _NOISY[folder]:
        moved = plain.forward(cases.config_of(folder), noisy, ids) - want
        moved = moved - moved.mean(dim=-1, keepdim=True)
        worst = torch.maximum(worst, moved.pow(2).mean(dim=-1).sqrt() / want.std(dim=-1, unbiased=False))
    return worst


def _close(got, want, dtype, what, folder=None, ids=None):
    """Row by row: the root mean square of the difference over the vocabulary (mean taken off) as a share of the row's
    spread: at most 5e-5 in float32, 5 % in bfloat16 or one and a half times what rounding alone moves that row by if that
    is more (``_what_rounding_does``), and no single value off by more than four times that."""
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} vs {tuple(want.shape)}"
    diff = got - want
    diff = diff - diff.mean(dim=-1, keepdim=True)
    spread = want.std(dim=-1, unbiased=False)
    rms, top = diff.pow(2).mean(dim=-1).sqrt() / spread, diff.abs().max(dim=-1).values / spread
    bound = torch.full_like(rms, 5e-5 if dtype == torch.float32 else 0.05)
    if dtype == torch.bfloat16 and folder is not None and not bool((rms <= bound).all() and (top <= 4 * bound).all()):
        bound = torch.maximum(bound, 1.5 * _what_rounding_does(folder, ids))
    worst = int(torch.argmax(rms / bound))
    assert bool((rms <= bound).all()) and bool((top <= 4 * bound).all()), \
        f"{what}: row {worst} of {len(rms)}: rms error {float(rms[worst]):.3g} of the spread (bound {float(bound[worst]):.3g}), largest {float(top.max()):.3g}"


def _check(folder, dtype, requests, got, what):
    for tag, req in requests.items():
        _close(got[tag], _expected(folder, req.ids), dtype, f"{what} request {tag}", folder, req.ids)


def _near(got, want, dtype, what, atol=None, rtol=None):
    a, r = (2e-5, 2e-5) if dtype == torch.float32 else (3e-2, 2e-2)
    a, r = (atol if atol is not None else a), (rtol if rtol is not None else r)
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    err = (got - want).abs()
    bound = a + r * want.abs()
    assert bool((err <= bound).all()), f"{what}: max error {float(err.max()):.3g}, over its bound by {float((err - bound).max()):.3g}"


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ================================================================================================ kernels alone
def _run_recurrence(dtype, d, dv, heads, tau, pieces_per_row, slots, seed, chunks, strong=1.0):
    """Rows fed in the given pieces (a list of token counts per row, step by step) through the walk over tokens or the
    chunked form; returns what was read, what the plain recurrence gives, and the rows' states after."""
    from kestrel_amd.ops import core, fast

    gen = torch.Generator().manual_seed(seed)
    H = heads
    n_slots = 5
    before, behind = 12, H * d * dv + 4                              # a slot's state lies in a wider row
    wide = torch.zeros(n_slots + 1, before + behind, device=DEV)
    wide[n_slots].fill_(float("nan"))                                # the spare row is nobody's
    wide[:, :before].fill_(7.0)
    state = wide[:, before:before + H * d * dv]
    data = [torch.randn(sum(p), 8 + H * (2 * d + dv), generator=gen).to(dtype) for p in pieces_per_row]
    # decays between almost 1 and next to nothing, channel by channel
    pre = [torch.randn(sum(p), H * d, generator=gen) * 2 * strong + torch.linspace(-6 * strong, 6, H * d)[None, :] for p in pieces_per_row]
    offsets = (8, 8 + H * d, 8 + 2 * H * d)                          # the projected rows lie in wider ones
    q_scale = d ** -0.5
    got = [[] for _ in data]
    at = [0] * len(data)
    for step in range(max(len(p) for p in pieces_per_row)):
        rows = [i for i, p in enumerate(pieces_per_row) if step < len(p)]
        counts = [pieces_per_row[i][step] for i in rows]
        projected = torch.cat([data[i][at[i]:at[i] + c] for i, c in zip(rows, counts)]).to(DEV)
        z = torch.cat([pre[i][at[i]:at[i] + c] for i, c in zip(rows, counts)]).to(DEV)
        n = projected.shape[0]
        cu = [0]
        for c in counts:
            cu.append(cu[-1] + c)
        raw = torch.full((n, H * dv), float("nan"), device=DEV)
        operands = (projected, offsets, z, tau, q_scale, state, _i32(cu), _i32([slots[i] for i in rows]), raw, H, d, dv)
        if chunks:
            scratch = torch.full((fast.gated_chunks_scratch(n, len(rows), H, d, dv),), float("nan"), device=DEV)
            assert fast.gated_chunks_bf16(*operands, scratch)
        else:
            core.gated_linear_attention(*operands)
        for j, (i, c) in enumerate(zip(rows, counts)):
            got[i].append(raw[cu[j]:cu[j + 1]].double().cpu())
            at[i] += c
    want, states = [], []
    for x, z in zip(data, pre):
        x = x.double()
        n = x.shape[0]
        q, k = (x[:, o:o + H * d].reshape(n, H, d) for o in offsets[:2])
        v = x[:, offsets[2]:offsets[2] + H * dv].reshape(n, H, dv)
        alpha = plain.decays(z.double(), tau).reshape(n, H, d)
        want.append(plain.gated_sum(q * q_scale, k, v, alpha).reshape(n, -1))
        last = torch.zeros(H, d, dv, dtype=F64)
        for t in range(n):
            last = alpha[t][:, :, None] * last + k[t][:, :, None] * v[t][:, None, :]
        states.append(last.transpose(1, 2))
    return [torch.cat(p) for p in got], want, wide, state, states


PIECES = [[150], [1] * 7, [17, 2, 0, 33, 1, 1, 40], [0, 0, 3, 0, 1], [5, 5]]
SLOTS = [0, 1, 2, 3, -1]


def _check_recurrence(dtype, d, dv, heads, chunks, tau=4.0, strong=1.0):
    got, want, wide, state, states = _run_recurrence(dtype, d, dv, heads, tau, PIECES, SLOTS, d + dv, chunks, strong)
    for row, (a, b) in enumerate(zip(got, want)):
        if SLOTS[row] < 0:
            assert float(a.abs().max()) == 0.0, "a row without a request reads zeros"
            continue
        # (a read-out is a long sum: an error is measured against the row's size; neither form rounds keys, queries or values)
        size = float(b.pow(2).mean().sqrt())
        rtol = 1e-5 if dtype == torch.float32 else 1e-4
        assert float((a - b).abs().max()) <= 6 * rtol * size + rtol * float(b.abs().max()), \
            f"{d} x {dv} row {row}: error {float((a - b).abs().max()):.3g} at size {size:.3g}"
        kept = state[SLOTS[row]].double().cpu().view_as(states[row])
        assert float((kept - states[row]).abs().max()) <= rtol * (float(states[row].abs().max()) + 1), f"{d} x {dv} row {row}: state"
    assert bool(torch.isnan(state[5]).all()), "the spare row is left alone"
    assert bool((wide[:5, :12] == 7.0).all()) and bool((wide[:5, 12 + heads * d * dv:] == 0.0).all()), "what lies beside a state is left alone"


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("d, dv, heads", [(16, 16, 3), (64, 40, 5), (10, 7, 2), (1, 3, 2), (30, 64, 4), (128, 80, 2), (100, 33, 1),
                                           (256, 24, 2), (300, 20, 1), (512, 8, 1)])
def test_recurrence_token_by_token(d, dv, heads, dtype):
    """Rows of 1 to 150 tokens cut into a prompt, portions and single tokens, beside a row without a request; key heads that
    fill a group of lanes, part of one, and several loads a lane; channels that forget at once, slowly and hardly at all."""
    _check_recurrence(dtype, d, dv, heads, False)


def test_recurrence_with_many_workgroups():
    """As many rows as make a group of lanes take four value channels."""
    got, want, *_rest = _run_recurrence(torch.float32, 32, 40, 5, 2.0, [[2, 1]] * 4 + [[3]] * 200, [0, 1, 2, 3] + [-1] * 200, 3, False)
    for row in range(4):
        _near(got[row], want[row], torch.float32, f"row {row}")


@pytest.mark.parametrize("d, dv, heads", [(16, 16, 3), (64, 64, 5), (32, 40, 4), (48, 8, 2), (128, 80, 2), (96, 136, 2), (224, 24, 1)])
def test_recurrence_by_chunks_on_the_matrix_cores(d, dv, heads):
    """The same rows through the three launches over chunks: chunks that are full, that end early, in every block, rows of
    several chunks."""
    _check_recurrence(torch.bfloat16, d, dv, heads, True)


@pytest.mark.parametrize("chunks", [False, True], ids=["walk", "chunks"])
def test_decays_that_leave_nothing(chunks):
    """tau below 1 and pre-activations down to -90: products of decays far below the smallest number, inside a block, between
    blocks and between chunks, beside channels that keep nearly everything."""
    _check_recurrence(torch.bfloat16, 64, 32, 3, chunks, tau=0.25, strong=15.0)


def test_many_rows_of_chunks():
    """More rows than a wave looks at at a time when a workgroup finds its chunk."""
    counts = [1 + (i * 37) % 90 for i in range(140)]
    slots = [i if i < 5 else -1 for i in range(140)]
    got, want, *_rest = _run_recurrence(torch.bfloat16, 32, 16, 2, 8.0, [[c] for c in counts], slots, 9, True)
    for row in range(140):
        if slots[row] >= 0:
            _near(got[row], want[row], torch.bfloat16, f"row {row}", atol=1e-3, rtol=1e-3)
        else:
            assert float(got[row].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("d, dv, heads, rank", [(64, 128, 3, 64), (16, 16, 1, 5), (4, 7, 2, 1), (36, 20, 5, 9), (128, 96, 2, 32), (256, 24, 1, 16), (100, 300, 2, 130),
                                                 (224, 512, 1, 1000)])
def test_a_token_of_the_recurrence_in_one_launch(d, dv, heads, rank, dtype):
    """Four tokens in a row of three requests and a row without one, from the projected rows to the gated heads; the state goes
    through three slots of wider rows, the output into columns of wider rows."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(d + dv)
    H, tau, eps = heads, 0.7, 1e-4
    a2 = (torch.randn(H * d, rank, generator=gen) / math.sqrt(rank)).to(dtype)
    bias, gain = torch.randn(H * d, generator=gen), 1 + 0.3 * torch.randn(dv, generator=gen)
    wide = torch.full((5, 4 + H * d * dv + 4), 7.0, device=DEV)
    state = wide[:, 4:4 + H * d * dv]
    state.fill_(float("nan"))
    slots = [2, 0, -1, 3]
    state[[2, 0, 3]] = 0.0
    columns = 3 + 2 * H * d + 2 * H * dv + rank
    rows = torch.randn(4, 4, columns, generator=gen).to(dtype)                 # [token, row]
    offsets = [3, 3 + H * d, 3 + 2 * H * d, 3 + 2 * H * d + H * dv, 3 + 2 * H * d + 2 * H * dv]
    got = []
    for x in rows:
        out = torch.full((4, H * dv + 5), 7.0, dtype=dtype, device=DEV)
        assert core.gated_step(x.to(DEV), offsets, a2.to(DEV), bias.to(DEV), gain.to(DEV), tau, 0.3, eps, state, _i32(slots), out[:, 5:], H, d, dv)
        assert bool((out[:, :5] == 7.0).all())
        got.append(out[:, 5:].double().cpu())
    for r, slot in enumerate(slots):
        x = rows[:, r].double()
        q, k = (x[:, o:o + H * d].reshape(4, H, d) for o in offsets[:2])
        v, gate = (x[:, o:o + H * dv].reshape(4, H, dv) for o in offsets[2:4])
        alpha = plain.decays(x[:, offsets[4]:] @ a2.double().T + bias.double(), tau).reshape(4, H, d)
        want = (plain.rms(plain.gated_sum(q * 0.3, k, v, alpha), eps) * gain.double() * plain.silu(gate)).reshape(4, -1)
        if slot < 0:
            want = torch.zeros_like(want)
        _near(torch.stack([g[r] for g in got]), want, dtype, f"row {r}", atol=1e-4 if dtype == torch.float32 else 2e-3, rtol=1e-4 if dtype == torch.float32 else 1e-2)
    assert bool(torch.isnan(state[[1, 4]]).all()) and bool((wide[:, :4] == 7.0).all()) and bool((wide[:, 4 + H * d * dv:] == 7.0).all())


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("heads, dv", [(1, 4), (3, 7), (5, 64), (2, 128), (4, 33), (1, 300)])
def test_norm_of_every_head_with_one_gain_kernel(heads, dv, dtype):
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(dv)
    n = 5
    raw = torch.randn(n, heads * dv, generator=gen) * torch.tensor([1.0, 1e-3, 30.0, 0.0, 2.0])[:, None]
    raw[0, :dv] *= 50                                                # (a head's size must not touch the others')
    gain = 1 + 0.3 * torch.randn(dv, generator=gen)
    gate = torch.randn(n, heads * dv + 12, generator=gen).to(dtype)  # columns of wider rows
    wide = torch.full((n, heads * dv + 8), 7.0, dtype=dtype, device=DEV)
    core.heads_rmsnorm(raw.to(DEV), gain.to(DEV), gate.to(DEV)[:, 12:], wide[:, 8:], heads, dv, 1e-4)
    want = (plain.rms(raw.double().view(n, heads, dv), 1e-4) * gain.double()).reshape(n, -1) * plain.silu(gate[:, 12:].double())
    _near(wide[:, 8:], want, dtype, "heads", rtol=1e-2 if dtype == torch.bfloat16 else 1e-5, atol=1e-6)
    assert bool((wide[:, :8] == 7.0).all())


STREAM_SIZES = [(1, 48), (2, 256), (3, 128), (4, 1000), (4, 4096), (4, 9000), (5, 100), (7, 64), (16, 36), (3, 70)]


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("streams, dim", STREAM_SIZES)
def test_streams_between_two_sublayers_kernel(streams, dim, dtype):
    """Begun from the embedding, read; written and read; written alone; chosen rows read through the final norm."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(dim + streams)
    n = 7
    embedded, y = torch.randn(n, dim, generator=gen) * 3, torch.randn(n, dim, generator=gen)
    mix, out, into = torch.randn(streams, streams, generator=gen), torch.randn(streams, generator=gen), torch.randn(streams, generator=gen)
    gain = 1 + 0.3 * torch.randn(dim, generator=gen)
    on = lambda t: t.to(DEV)  # noqa: E731
    form = ("layernorm", on(gain), None, 1e-3)
    x = torch.full((n, streams, dim), float("nan"), device=DEV)
    h = torch.full((n, dim), float("nan"), dtype=dtype, device=DEV)
    rows = dict(rtol=1e-2 if dtype == torch.bfloat16 else 2e-5, atol=2e-5 if dtype == torch.float32 else 1e-3)

    def read(X, a):
        return plain.layer_norm(plain.read_streams(X, a.double()), gain.double(), 1e-3)

    core.streams_step(x, embedded=on(embedded), reading=(on(into), form), h=h)
    X = embedded.double()[None].repeat(streams, 1, 1)
    assert torch.equal(x.cpu(), embedded[:, None].repeat(1, streams, 1))
    _near(h, read(X, into), dtype, "first reading", **rows)
    core.streams_step(x, on(y), on(mix), on(out), (on(into), form), h)
    X = plain.write_streams(X, mix.double(), out.double(), y.double())
    _near(x.transpose(0, 1), X, torch.float32, "streams", atol=1e-4)
    _near(h, read(X, into), dtype, "second reading", **rows)
    core.streams_step(x, on(y), on(mix.T.contiguous()), on(out))
    X = plain.write_streams(X, mix.T.double(), out.double(), y.double())
    _near(x.transpose(0, 1), X, torch.float32, "written alone", atol=4e-4)
    chosen = [5, 0, 5]
    last = torch.full((3, dim), float("nan"), dtype=dtype, device=DEV)
    core.streams_step(x, reading=(None, form), h=last, rows=_i32(chosen))
    _near(last, read(X, torch.ones(streams))[chosen], dtype, "the sum of chosen rows", rtol=1e-2 if dtype == torch.bfloat16 else 1e-4, atol=1e-4 if dtype == torch.float32 else 1e-3)
    core.streams_step(x, reading=(on(into), ("rms", on(gain), None, 1e-3)), h=h)
    _near(h, plain.rms(plain.read_streams(X, into.double()), 1e-3) * gain.double(), dtype, "through a root mean square",
          rtol=1e-2 if dtype == torch.bfloat16 else 1e-4, atol=1e-4 if dtype == torch.float32 else 1e-3)


@pytest.mark.parametrize("outputs, top, groups, keep", [(10, 2, 2, 1), (8, 3, 4, 2), (5, 1, 0, 0), (64, 8, 8, 3), (200, 6, 10, 4),
                                                         (3, 3, 1, 1), (3, 2, 3, 2), (512, 4, 64, 2), (1, 1, 1, 1)])
def test_choice_by_sigmoids_and_pairs_of_scores_kernel(outputs, top, groups, keep):
    """Groups that count by their two largest choice scores (by one, where a group has one), corrections that make choice
    scores negative and that the weights leave out; with and without a last choice that every token makes."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(outputs + top)
    n = 37
    logits = torch.randn(n, outputs + 1, generator=gen) * 2
    correction = torch.randn(outputs, generator=gen) * 0.4 - 1.0
    want_i, want_w = plain.routing(logits[:, :outputs].double(), correction.double(), top, (groups, keep) if groups else None)
    for always in (None, outputs):
        columns = top + (always is not None)
        chosen = torch.full((n, columns), -1, dtype=torch.int32, device=DEV)
        weights = torch.zeros(n, columns, device=DEV)
        core.route(logits.to(DEV), outputs, correction.to(DEV), top, groups, keep, 1.0, chosen, weights, scores="sigmoid", group_best=2, always=always)
        assert torch.equal(chosen[:, :top].cpu().long(), want_i)
        _near(weights[:, :top], want_w, torch.float32, "weights", atol=1e-6)
        if always is not None:
            assert bool((chosen[:, top] == outputs).all()) and bool((weights[:, top] == 1.0).all())


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("n, dim, ff, n_experts, top, streams", [(3, 100, 36, 5, 2, 5), (70, 128, 48, 6, 3, 4), (200, 64, 96, 4, 1, 2), (150, 192, 80, 33, 4, 3),
                                                                  (90, 16, 176, 3, 2, 1), (64, 2048, 704, 31, 5, 4), (6, 72, 24, 4, 4, 3), (100, 40, 8, 1, 1, 2)])
def test_clamped_experts_and_the_streams_they_are_written_into(n, dim, ff, n_experts, top, streams, dtype):
    """Experts with clamps that bite on about every second number, pair by pair and (bfloat16) listed by expert; their weighted
    sum with a shared expert's output written into the streams and read again."""
    from kestrel_amd.engine.batch import Workspace
    from kestrel_amd.ops import core, fast
    from kestrel_amd.ops.linear import ACT_GATED, activation_code, pair_rows
    from kestrel_amd.parts.specs import GateClamp

    gen = torch.Generator().manual_seed(n + dim)
    limit = 0.7
    h = torch.randn(n, dim, generator=gen).to(dtype)
    gate, up = ((torch.randn(n_experts, ff, dim, generator=gen) / math.sqrt(dim)).to(dtype) for _ in range(2))
    down = (torch.randn(n_experts, dim, ff, generator=gen) / math.sqrt(ff)).to(dtype)
    chosen = torch.stack([torch.randperm(n_experts, generator=gen)[:top] for _ in range(n)]).to(torch.int32)
    weights, shared = torch.rand(n, top, generator=gen), torch.randn(n, dim, generator=gen)
    w = {}
    for e in range(n_experts):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = gate[e].double(), up[e].double(), down[e].double()
    y = torch.stack([sum(float(weights[t, k]) * plain.expert(h[t:t + 1].double(), w, f"e{int(chosen[t, k])}", limit)[0] for k in range(top))
                     for t in range(n)]) + shared.double()
    pairs_w = torch.stack([pair_rows(gate[e], up[e]) for e in range(n_experts)]).to(DEV)
    act, clamp = activation_code("silu") | ACT_GATED, GateClamp(limit, 1.702, 1.0)
    hidden = torch.zeros(n * top, ff, dtype=dtype, device=DEV)
    pairs = torch.full((n * top, dim), float("nan"), device=DEV)
    flat = chosen.to(DEV).view(-1)
    core.experts_linear(h.to(DEV), top, pairs_w, flat, hidden, act, clamp=clamp)
    core.experts_linear(hidden, 1, down.to(DEV), flat, pairs)
    X = torch.randn(streams, n, dim, generator=gen)
    mix, out, into = torch.randn(streams, streams, generator=gen), torch.randn(streams, generator=gen), torch.rand(streams, generator=gen) + 0.2
    gain = 1 + 0.2 * torch.randn(dim, generator=gen)
    want = plain.write_streams(X.double(), mix.double(), out.double(), y)
    normed = plain.layer_norm(plain.read_streams(want, into.double()), gain.double(), 1e-5)

    def written(pairs, what):
        x = X.transpose(0, 1).contiguous().to(DEV)
        rows = torch.full((n, dim), float("nan"), dtype=dtype, device=DEV)
        core.streams_experts(x, pairs, h.to(DEV), chosen.to(DEV), weights.to(DEV), n_experts, shared.to(DEV), None, mix.to(DEV), out.to(DEV),
                             (into.to(DEV), ("layernorm", gain.to(DEV), None, 1e-5)), rows)
        _near(x.transpose(0, 1), want, dtype, what, atol=1e-4 if dtype == torch.float32 else 6e-2)
        _near(rows, normed, dtype, what + ", read", atol=2e-4 if dtype == torch.float32 else 8e-2)

    written(pairs, "pair by pair")
    if dtype == torch.bfloat16 and dim % 16 == 0 and ff % 16 == 0:
        pairs = torch.full((n * top, dim), float("nan"), device=DEV)
        assert fast.experts_feed_forward_bf16(h.to(DEV), pairs_w, down.to(DEV), chosen.to(DEV), None, pairs, act, Workspace(torch.device(DEV)), clamp=clamp)
        written(pairs, "by expert")
    if dtype == torch.bfloat16 and dim % 8 == 0 and ff % 8 == 0 and n * top <= 512:
        pairs = torch.full((n * top, dim), float("nan"), device=DEV)
        assert fast.experts_few_bf16(h.to(DEV), pairs_w, down.to(DEV), chosen.to(DEV), torch.zeros_like(hidden), pairs, act, clamp=clamp)
        written(pairs, "few pairs")


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("heads, kv_heads, hd, hdv, taps, rot, ps", [
    (4, 2, 32, 64, 4, 16, 16), (2, 2, 64, 32, 3, 64, 16), (8, 1, 16, 8, 2, 8, 16), (3, 1, 12, 10, 5, 6, 4), (2, 1, 128, 128, 4, 128, 16),
    (1, 1, 256, 16, 1, 32, 16), (5, 5, 48, 24, 4, 48, 16), (40, 8, 64, 64, 4, 32, 16), (2, 1, 32, 24, 6, 32, 16), (2, 2, 32, 32, 4, 32, 4)])
def test_convolution_norm_rotation_and_cache_write_kernel(heads, kv_heads, hd, hdv, taps, rot, ps, dtype):
    """A sequence of 75 tokens in portions (shorter than the taps, across pages, whole pages, one token) beside another row and
    a padding token; with the lists of runs that a step brings and without them; the state lies in a wider row."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(hd + taps)
    channels = (heads + kv_heads) * hd + kv_heads * hdv
    n, base = 75, 50.0
    u, other = torch.randn(n, channels, generator=gen).to(dtype), torch.randn(40, channels, generator=gen).to(dtype)
    w = torch.randn(channels, taps, generator=gen)
    freqs = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float32, device=DEV)
    own = max(taps - 1, 1) * channels
    for with_runs in (True, False):
        wide = torch.full((4, own + 8), 7.0, device=DEV)
        state = wide[:, 4:4 + own].unflatten(1, (max(taps - 1, 1), channels))
        state.fill_(float("nan"))
        state[[1, 3]] = 0.0                                   # (the cache manager clears a slot when a request is admitted)
        pages = -(-n // ps) + 4
        k_cache = torch.zeros(pages, kv_heads, ps, hd, dtype=dtype, device=DEV)
        v_cache = torch.zeros(pages, kv_heads, hdv, ps, dtype=dtype, device=DEV)
        order = torch.randperm(pages, generator=gen).tolist()
        q_rows, at, beside = [], 0, 0
        for count, extra in ((1, 1), (4, 0), (2, 3), (1, 1), (34, 2), (16, 0), (1, 1), (1, 1), (15, 5)):
            single = count == 1 and extra == 1
            pad = 0 if single else 1                          # a padding token: no row's, cached nowhere
            rows = torch.cat([u[at:at + count], other[beside:beside + extra], other[:pad]])
            m = rows.shape[0]
            places = list(range(at, at + count)) + list(range(beside, beside + extra)) + [0] * pad
            slots = [order[p // ps] * ps + p % ps for p in range(at, at + count)] + [-1] * (extra + pad)
            first, counts = [], []
            for t in range(m):
                if t == 0 or slots[t] < 0 or slots[t - 1] < 0 or slots[t] % ps == 0 or t == count:
                    first.append(t)
                    counts.append(0)
                counts[-1] += 1
            q_out = torch.full((m, heads * hd), float("nan"), dtype=dtype, device=DEV)
            core.conv_prepare(rows.to(DEV), w.to(DEV), state if taps > 1 else None, _i32([0, count, count + extra, m]) if not single else _i32([0, 1, 2]),
                              _i32([1, 3, -1]) if not single else _i32([1, 3]), _i32([0] * count + [1] * extra + [2] * pad), _i32(places), _i32(slots),
                              q_out, k_cache, v_cache, heads, kv_heads, hd, kv_heads, hdv, ps, freqs, "halves", unit_norm_eps=1e-4,
                              runs=(_i32(first + [0]), _i32(counts + [0])) if with_runs else None, single_tokens=single)
            q_rows.append(q_out[:count].double().cpu())
            at += count
            beside += extra
        y = plain.causal_conv(u.double(), w.double())
        turn = lambda x: plain.rms(plain.rotate_halves(x, rot, base), 1e-4)  # noqa: E731
        q, k = turn(y[:, :heads * hd].reshape(n, heads, hd)), turn(y[:, heads * hd:(heads + kv_heads) * hd].reshape(n, kv_heads, hd))
        v = y[:, (heads + kv_heads) * hd:].reshape(n, kv_heads, hdv)
        tol = dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
        flat = [order[p // ps] * ps + p % ps for p in range(n)]
        _near(torch.cat(q_rows).view(n, heads, hd), q, dtype, "queries", **tol)
        _near(k_cache.permute(0, 2, 1, 3).reshape(-1, kv_heads, hd)[flat], k, dtype, "keys", **tol)
        _near(v_cache.permute(0, 3, 1, 2).reshape(-1, kv_heads, hdv)[flat], v, dtype, "values", **tol)
        untouched = torch.ones(pages * ps, dtype=torch.bool)
        untouched[flat] = False
        assert float(k_cache.permute(0, 2, 1, 3).reshape(pages * ps, -1)[untouched.to(DEV)].abs().max()) == 0.0
        if taps > 1:
            _near(state[1], u.double()[n - taps + 1:], torch.float32, "state")
            _near(state[3], other.double()[beside - taps + 1:beside], torch.float32, "the other row's state")
            assert bool(torch.isnan(state[[0, 2]]).all())
        assert bool((wide[:, :4] == 7.0).all()) and bool((wide[:, 4 + own:] == 7.0).all())


def test_branches_that_run_as_one_and_branches_that_do_not():
    """The mixer with its two branches' linears joined gives what the branches give one by one (weights that some fp32 constant of
    a branch takes up, and weights that none does)."""
    from kestrel_amd.parts.base import build_part
    from kestrel_amd.models import gozatar

    for name, joined in (("P", [True] * 4), ("Q", [True, False, True, True])):
        plan = gozatar.build_plan(gozatar.GozatarConfig.from_dict(cases.CONFIGS[name]))
        for layer, want in zip(plan.layers, joined):
            part = build_part("mixer", layer.mixer)
            gen = torch.Generator().manual_seed(1)
            tensors = {k: (torch.randn(p.shape, generator=gen) * 0.1).to(DEV) for k, p in part.params().items()}
            gain = tensors["1.norm.weight"].clone()
            part.bind(tensors, torch.float32, torch.device(DEV))
            assert (part.in_weight is not None) == want
            kept = part.branches[1].gain
            assert torch.equal(kept, gain * float(layer.mixer.weights[1]) if want else gain)


def test_the_matrix_core_kernels_run_where_sizes_allow():
    """In bfloat16 the models whose sizes the matrix-core kernels take run them for prompts."""
    from kestrel_amd.ops import fast

    calls = {}
    names = ("gated_chunks_bf16", "experts_few_bf16", "experts_feed_forward_bf16")
    originals = {name: getattr(fast, name) for name in names}

    def spy(name):
        def call(*args, **kwargs):
            done = originals[name](*args, **kwargs)
            calls.setdefault(name, []).append(done)
            return done
        return call

    for name in names:
        setattr(fast, name, spy(name))
    try:
        for model in ("P", "R"):
            calls.clear()
            folder = cases.model_dir(model)
            for length in (70, 270):             # (too few pairs of a token and an expert for lists, and enough)
                helpers.replay(_runner(folder, torch.bfloat16), {"r": Request("r", _ids(folder, 900, length))}, [[("r", length)]])
            assert set(calls) == set(names) and all(bool(d) for done in calls.values() for d in done), (model, calls)
    finally:
        for name in names:
            setattr(fast, name, originals[name])


# ================================================================================================ the model, cut every way
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_every_layer(name, dtype):
    """The sum of the streams after every layer, then the logits."""
    from kestrel_amd.parts.block import Block

    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype)
    ids = _ids(folder, 1, 45)
    seen = []
    original = Block.forward

    def spy(self, x, *args, **kwargs):
        result = original(self, x, *args, **kwargs)
        seen.append(x.detach().double().cpu().sum(dim=1))
        return result

    Block.forward = spy
    try:
        got = helpers.replay(runner, {"r": Request("r", ids)}, [[("r", len(ids))]])
    finally:
        Block.forward = original
    streams = []
    want = plain.forward(cases.config_of(folder), cases.stored_weights(folder), ids, streams)
    assert len(seen) == len(streams)
    apart = lambda a, b: ((a - b).pow(2).mean(dim=-1) / b.pow(2).mean(dim=-1)).sqrt()  # noqa: E731
    bounds = [torch.full((len(ids),), 2e-5 if dtype == torch.float32 else 3e-2, dtype=F64) for _ in streams]
    if dtype == torch.bfloat16:                     # (or what rounding alone moves the row by, ``_what_rounding_does``)
        gen = torch.Generator().manual_seed(98)
        for _ in range(3):
            moved = []
            plain.forward(cases.config_of(folder), {k: v.double() * (1 + 2.0 ** -8 * torch.randn(v.shape, generator=gen, dtype=F64))
                                                    for k, v in cases.stored_weights(folder).items()}, ids, moved)
            bounds = [torch.maximum(bound, apart(a, b)) for bound, a, b in zip(bounds, moved, streams)]
    for layer, (a, b, bound) in enumerate(zip(seen, streams, bounds)):
        over = apart(a, b) / bound
        assert float(over.max()) <= 1.0, f"{name} layer run {layer}: row {int(over.argmax())} is {float(over.max()):.3g} times its bound away"
    _close(got["r"], want, dtype, f"{name} logits", folder, ids)


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(name, dtype):
    """Each request alone and whole: the first tokens of a sequence (1, 2, 3), lengths around a page's, a window's and a
    chunk's edges, and well beyond every window."""
    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype)
    for seed, length in enumerate([1, 2, 3, 7, 8, 16, 17, 24, 25, 33, 40, 41, 63, 64, 65, 129, 260]):
        reqs = {"r": Request("r", _ids(folder, 100 + seed, length))}
        _check(folder, dtype, reqs, helpers.replay(runner, reqs, [[("r", length)]]), f"{name} whole {length}")


@pytest.mark.parametrize("graphs", [False, True], ids=["launched", "graphs"])
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_then_token_by_token(name, dtype, graphs):
    """Most of the request in one step, then one token a step across the window's edge; and a request decoded from its very
    first token."""
    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype, graphs=graphs)
    for seed, (length, head) in enumerate([(150, 60), (70, 1), (48, 47)]):
        reqs = {"r": Request("r", _ids(folder, 200 + seed, length))}
        got = helpers.replay(runner, reqs, [[("r", head)]] + [[("r", 1)]] * (length - head))
        _check(folder, dtype, reqs, got, f"{name} decode {length}/{head}")
    assert (runner.graph_replays > 0) == graphs


@pytest.mark.parametrize("graphs", [False, True], ids=["launched", "graphs"])
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_portions_of_changing_size(name, dtype, graphs):
    """Portions cut anywhere: in the middle of a page, a window and a chunk, down to two tokens."""
    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype, graphs=graphs)
    for seed, cuts in enumerate([[2, 2, 3, 9, 16, 1, 31, 2, 40, 5, 64, 2], [17, 2, 2, 2, 50], [33, 32, 31, 7], [130, 65, 2]]):
        reqs = {"r": Request("r", _ids(folder, 300 + seed, sum(cuts)))}
        _check(folder, dtype, reqs, helpers.replay(runner, reqs, [[("r", c)] for c in cuts]), f"{name} portions {seed}")


@pytest.mark.parametrize("graphs", [False, True], ids=["launched", "graphs"])
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_in_reused_pages_and_slots(name, dtype, graphs):
    """Up to four live requests of unequal lengths, portions of some beside single tokens of others, in a pool so small
    that pages and state slots are used again (what is given back is filled with NaN first); every request must come
    out as it does alone."""
    folder = cases.folder_for(name, dtype)
    lengths = {"a": 90, "b": 37, "c": 61, "d": 5, "e": 130, "f": 44, "g": 2}
    runner = _runner(folder, dtype, n_pages=24, max_requests=4, graphs=graphs)
    reqs = {tag: Request(tag, _ids(folder, 400 + i, n)) for i, (tag, n) in enumerate(lengths.items())}
    steps = [[("a", 50), ("b", 20)], [("a", 1), ("b", 17), ("c", 30)], [("a", 1), ("c", 2), ("d", 5)],
             [("a", 38), ("c", 29)],                                  # a, c and d end; b ended before
             [("e", 64), ("f", 3)], [("e", 1), ("f", 41), ("g", 2)], [("e", 1)], [("e", 62)], [("e", 1)], [("e", 1)]]
    got = helpers.replay(runner, reqs, steps, poison=True)
    _check(folder, dtype, reqs, got, f"{name} mixed")
    assert runner.cache.free_slots == 4


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_replayed_steps_of_any_shape(name, dtype):
    """Steps replayed as graphs, one graph serving steps of different make-up in turn: long portions alone, beside short ones and
    single tokens; in pages that were given back and hold NaN."""
    from tests.test_mixed_graphs_gpu import replay_last_places

    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype, n_pages=40, max_requests=8, graphs=True)
    assert runner.mixed_graphs
    lengths = {"a": 190, "b": 112, "c": 150, "d": 75, "e": 128, "f": 120, "g": 70, "h": 66}
    steps = [[("a", 100), ("b", 20)],                              # all but the last: 65 to 128 tokens, the same graph
             [("a", 1), ("b", 60), ("c", 50)],                     # no portion long enough
             [("a", 64), ("b", 1), ("c", 2), ("d", 60)],           # one just long enough
             [("a", 1), ("c", 98), ("d", 15)],
             [("a", 24), ("b", 31), ("e", 63)],                    # a, b end; one token short of long
             [("e", 65), ("f", 55)],
             [("f", 65), ("g", 2)],
             [("g", 68)],
             [("h", 66)]]
    reqs = {tag: Request(tag, _ids(folder, 800 + i, n)) for i, (tag, n) in enumerate(lengths.items())}
    got = replay_last_places(runner, reqs, steps, wanted=2)
    assert runner.mixed_graph_replays == len(steps) and len(runner._mixed) == 1, sorted(runner._mixed)
    for tag, req in reqs.items():
        places = sorted(got[tag])
        want = _expected(folder, req.ids)
        bound = None
        if dtype == torch.bfloat16:
            bound = torch.clamp(_what_rounding_does(folder, req.ids)[places], min=0.05)
        diff = torch.stack([got[tag][p] for p in places]).double().cpu() - want[places]
        diff = diff - diff.mean(dim=-1, keepdim=True)
        rms = diff.pow(2).mean(dim=-1).sqrt() / want[places].std(dim=-1, unbiased=False)
        assert bool((rms <= (5e-5 if bound is None else bound)).all()), (name, tag, places, rms)


def test_a_slot_used_again_starts_from_nothing():
    """The cache manager clears a slot's state at admission: the second request in a slot must not see the first's."""
    folder = cases.model_dir("P")
    runner = _runner(folder, torch.float32, max_requests=1)
    for seed in (1, 2):
        reqs = {"r": Request("r", _ids(folder, 40 + seed, 30))}
        _check(folder, torch.float32, reqs, helpers.replay(runner, reqs, [[("r", 20)], [("r", 10)]]), f"use {seed}")


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
def test_long_decoding_under_graphs(dtype):
    """Three hundred tokens one by one beside a second request that comes and goes: the windows pass, their pages go back,
    the states are carried through every step."""
    folder = cases.folder_for("P", dtype)
    runner = _runner(folder, dtype, n_pages=24, max_requests=2, graphs=True)
    reqs = {"long": Request("long", _ids(folder, 500, 300)), "short": Request("short", _ids(folder, 501, 25))}
    steps = [[("long", 3)]] + [[("long", 1)]] * 100 + [[("long", 1), ("short", 20)]] + [[("long", 1), ("short", 1)]] * 5 \
        + [[("long", 1)]] * 191
    got = helpers.replay(runner, reqs, steps, poison=True)
    _check(folder, dtype, reqs, got, "long decoding")
    assert not runner.cache.live_slots


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
def test_a_far_key_and_the_windows_edges_in_the_model(dtype):
    """On a folder crafted so that it shows (``cases.crafted``; ``test_gozatar_cpu.py`` measures by how much): a token that
    calls and, at a chosen distance before it, the token it calls for: just inside and just outside either window, at a
    page's border, far back, and at the sequence's first place; inside a prompt, decoded alone, and with all but two tokens
    decoded."""
    base = cases.folder_for("P", dtype)
    folder = cases.crafted(base)
    windows = sorted({layer["mixer"]["left"]["mask"]["size"] for layer in cases.config_of(base)["layers"]}, reverse=True)
    length = 140
    at = length - 7
    edges = [w + e for w in windows for e in (-1, 0)]
    for distance in edges + [1, 16, 17, 2 * windows[0] + 5, at]:
        ids = list(range(10, 10 + length))
        ids[at], ids[at - distance] = cases.CALL, cases.ECHO
        want = _expected(folder, ids)
        for head in (len(ids), at - 3, 2):
            if head == 2 and distance not in (windows[0], at):
                continue
            runner = _runner(folder, dtype)
            reqs = {"r": Request("r", ids)}
            got = helpers.replay(runner, reqs, [[("r", head)]] + [[("r", 1)]] * (len(ids) - head))
            _close(got["r"], want, dtype, f"distance {distance}, prompt of {head}", folder, ids)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["P", "Q"])
def test_greedy_generation_through_the_entry_point(name, dtype):
    """Requests of different lengths submitted together through ``InferenceEngine``: the scheduler cuts prompts into
    portions beside the decoding of the others; with and without graphs, one and two steps in flight."""
    from kestrel_amd import InferenceEngine, RuntimeConfig

    folder = cases.folder_for(name, dtype)
    config, weights = cases.config_of(folder), cases.stored_weights(folder)
    prompts = [_ids(folder, 600 + i, n) for i, n in enumerate([5, 17, 33, 120])]
    n_new = 24
    slack = 1e-4 if dtype == "float32" else 8e-2
    for graphs, depth in ((False, 1), (True, 2)):
        engine = InferenceEngine.create_sync(RuntimeConfig(model_path=folder, dtype=dtype, max_batch_size=4, kv_cache_pages=40,
                                                           max_num_batched_tokens=96, enable_graphs=graphs, pipeline_depth=depth,
                                                           max_seq_len=160))
        try:
            results = engine.generate_batch_sync(prompts, max_new_tokens=n_new, temperature=0.0, stop_ids=())
        finally:
            engine.shutdown_sync()
        for prompt, result in zip(prompts, results):
            assert result.finish_reason == "length" and len(result.tokens) == n_new
            logits = plain.forward(config, weights, list(prompt) + list(result.tokens[:-1]))
            for i, token in enumerate(result.tokens):
                row = logits[len(prompt) - 1 + i]
                gap = float(row.max() - row[token])
                assert gap <= slack * max(1.0, float(row.std())), \
                    f"{name} {dtype} graphs={graphs}: token {i} is {token}, plain gives {int(row.argmax())} ({gap:.3g} better)"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program(dtype, tmp_path):
    """``bin/trace_run`` on a folder of this architecture: steps from standard input, logits into files, a request left out
    of a step, slots and pages used again."""
    folder = cases.folder_for("P", dtype)
    ids = {tag: _ids(folder, 700 + i, n) for i, (tag, n) in enumerate({"a": 40, "b": 9, "c": 70, "d": 3, "e": 21}.items())}
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": ids["a"][:30], "want": [0, 29]}, {"id": "b", "tokens": ids["b"], "want": [8]}], "end": ["b"]},
        {"step": 1, "entries": [{"id": "c", "tokens": ids["c"][:64], "want": []}, {"id": "d", "tokens": ids["d"], "want": [0, 1, 2]},
                                {"id": "e", "tokens": ids["e"][:2], "want": [1]}], "end": ["d"]},
        {"step": 2, "entries": [{"id": "c", "tokens": ids["c"][64:], "want": [5]}, {"id": "a", "tokens": ids["a"][30:], "want": [0, 9]},
                                {"id": "e", "tokens": ids["e"][2:], "want": [18]}], "end": ["a", "c", "e"]},
    ]
    out = tmp_path / "out"
    done = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                           "--max-tokens", "256"], input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                          capture_output=True, timeout=600, cwd=ROOT)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    full = {tag: _expected(folder, seq) for tag, seq in ids.items()}
    wanted = {0: [("a", 0), ("a", 29), ("b", 8)], 1: [("d", 0), ("d", 1), ("d", 2), ("e", 1)], 2: [("c", 69), ("a", 30), ("a", 39), ("e", 20)]}
    vocab = cases.config_of(folder)["vocab"]
    for step, places in wanted.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(places), vocab))
        want = torch.stack([full[tag][p] for tag, p in places])
        _close(got, want, torch.float32 if dtype == "float32" else torch.bfloat16, f"trace step {step}")


def test_command_line(tmp_path):
    """``python -m kestrel_amd random-weights`` from a configuration of this design, then ``generate`` on the folder."""
    env = dict(os.environ, PYTHONPATH=ROOT)
    config = tmp_path / "cfg.json"
    config.write_text(json.dumps(cases.CONFIGS["S"]))
    made = subprocess.run([sys.executable, "-m", "kestrel_amd", "random-weights", "--out", str(tmp_path / "m"), "--config", str(config),
                           "--seed", "5", "--std", "0.08", "--bias-std", "0.5", "--gain-std", "0.2"], capture_output=True, text=True,
                          env=env, cwd=ROOT)
    assert made.returncode == 0, made.stderr
    folder = str(tmp_path / "m")
    prompt = _ids(folder, 990, 9)
    done = subprocess.run([sys.executable, "-m", "kestrel_amd", "generate", "--model-path", folder, "--dtype", "float32",
                           "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "6", "--temperature", "0",
                           "--kv-cache-pages", "8", "--max-seq-len", "64"], capture_output=True, text=True, env=env, cwd=ROOT,
                          timeout=300)
    assert done.returncode == 0, done.stderr
    tokens = json.loads(done.stdout.strip().splitlines()[-1])["tokens"]
    logits = plain.forward(cases.config_of(folder), cases.stored_weights(folder), prompt + tokens[:-1])
    for i, token in enumerate(tokens):
        row = logits[len(prompt) - 1 + i]
        assert float(row.max() - row[token]) <= 1e-4 * max(1.0, float(row.std()))
