"""Vufolorn through the step function, the cache manager, the scheduler and the entry point, against the plain
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
from tests import vufolorn_cases as cases
from tests.helpers import Request
from tests.packed import CUTS, PackedStep
from tests.plain import vufolorn_plain as plain

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
    or two products ``q . k``, which may nearly cancel, and all heads are divided by their common root mean square."""
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
    spread: at most 5e-5 in float32, 4 % in bfloat16 or what rounding alone moves that row by if that is more
    (``_what_rounding_does``), and no single value off by more than four times that."""
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} vs {tuple(want.shape)}"
    diff = got - want
    diff = diff - diff.mean(dim=-1, keepdim=True)
    spread = want.std(dim=-1, unbiased=False)
    rms, top = diff.pow(2).mean(dim=-1).sqrt() / spread, diff.abs().max(dim=-1).values / spread
    bound = torch.full_like(rms, 5e-5 if dtype == torch.float32 else 0.04)
    if dtype == torch.bfloat16 and folder is not None and not bool((rms <= bound).all() and (top <= 4 * bound).all()):
        bound = torch.maximum(bound, _what_rounding_does(folder, ids))
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
def _run_recurrence(dtype, d, dv, decay, pieces_per_row, slots, seed, chunks):
    """Rows fed in the given pieces (a list of token counts per row, step by step) through the walk over tokens or the
    chunked form; returns what was read, what the plain recurrence gives, and the rows' states after."""
    from kestrel_amd.ops import core, fast
    from kestrel_amd.ops.linear import activation_code

    gen = torch.Generator().manual_seed(seed)
    H = len(decay)
    n_slots = 5
    pad = 8                                                          # the projected rows lie in wider ones
    state = torch.zeros(n_slots + 1, H * dv * d, device=DEV)
    state[n_slots].fill_(float("nan"))                               # the spare row is nobody's
    data = [torch.randn(sum(p), H * (2 * d + dv) + pad, generator=gen).to(dtype) for p in pieces_per_row]
    offsets = (0, H * d, 2 * H * d)
    decays = torch.tensor(decay, dtype=torch.float32, device=DEV)
    logs = torch.tensor([math.log2(a) for a in decay], dtype=torch.float32, device=DEV)
    got = [[] for _ in data]
    at = [0] * len(data)
    for step in range(max(len(p) for p in pieces_per_row)):
        rows = [i for i, p in enumerate(pieces_per_row) if step < len(p)]
        counts = [pieces_per_row[i][step] for i in rows]
        projected = torch.cat([data[i][at[i]:at[i] + c] for i, c in zip(rows, counts)]).to(DEV)
        n = projected.shape[0]
        cu = [0]
        for c in counts:
            cu.append(cu[-1] + c)
        raw = torch.full((n, H * dv), float("nan"), device=DEV)
        operands = (state, _i32(cu), _i32([slots[i] for i in rows]), raw, H, d, dv, activation_code("silu"))
        if chunks:
            need = fast.linear_attention_chunks_scratch(n, len(rows), H, d, dv)
            scratch = torch.full((need,), float("nan"), device=DEV)
            assert fast.linear_attention_chunks_bf16(projected, offsets, logs, *operands, scratch)
        else:
            core.linear_attention(projected, offsets, decays, *operands)
        for j, (i, c) in enumerate(zip(rows, counts)):
            got[i].append(raw[cu[j]:cu[j + 1]].double().cpu())
            at[i] += c
    want, states = [], []
    for x in data:
        x = plain.silu(x.double())
        n = x.shape[0]
        q, k = (x[:, o:o + H * d].reshape(n, H, d) for o in offsets[:2])
        v = x[:, offsets[2]:offsets[2] + H * dv].reshape(n, H, dv)
        want.append(plain.decayed_sum(q, k, v, decay).reshape(n, -1))
        last = torch.zeros(H, dv, d, dtype=F64)
        for h in range(H):
            weight = torch.tensor([decay[h] ** (n - 1 - t) for t in range(n)], dtype=F64)
            last[h] = (v[:, h] * weight[:, None]).T @ k[:, h]
        states.append(last)
    return [torch.cat(p) for p in got], want, state, states


PIECES = [[150], [1] * 7, [17, 2, 0, 33, 1, 1, 40], [0, 0, 3, 0, 1], [5, 5]]
SLOTS = [0, 1, 2, 3, -1]


def _check_recurrence(dtype, d, dv, decay, chunks):
    got, want, state, states = _run_recurrence(dtype, d, dv, decay, PIECES, SLOTS, seed=d + dv, chunks=chunks)
    for row, (a, b) in enumerate(zip(got, want)):
        if SLOTS[row] < 0:
            assert float(a.abs().max()) == 0.0, "a row without a request reads zeros"
            continue
        # (a read-out is a long sum: an error is measured against the row's size)
        size = float(b.pow(2).mean().sqrt())
        rtol = 1e-5 if dtype == torch.float32 else (8e-3 if chunks else 1e-4)
        assert float((a - b).abs().max()) <= 6 * rtol * size + rtol * float(b.abs().max()), \
            f"{d} x {dv} row {row}: error {float((a - b).abs().max()):.3g} at size {size:.3g}"
        kept = state[SLOTS[row]].double().cpu().view_as(states[row])
        assert float((kept - states[row]).abs().max()) <= rtol * (float(states[row].abs().max()) + 1), f"{d} x {dv} row {row}: state"
    assert bool(torch.isnan(state[5]).all()), "the spare row is left alone"


DECAYS = (0.9, 0.05, 0.9999, 1.0, 0.5)


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("d, dv, heads", [(16, 16, 3), (64, 40, 5), (10, 7, 2), (1, 3, 2), (30, 64, 4), (128, 80, 2), (100, 33, 1),
                                           (256, 24, 2), (300, 20, 1), (512, 8, 1)])
def test_recurrence_token_by_token(d, dv, heads, dtype):
    """Rows of 1 to 150 tokens cut into a prompt, portions and single tokens, beside a row without a request; key heads that
    fill a group of lanes, part of one, and several loads a lane; decays that forget at once, slowly and not at all."""
    _check_recurrence(dtype, d, dv, DECAYS[:heads], chunks=False)


def test_recurrence_with_many_workgroups():
    """As many rows as make a group of lanes take four value channels."""
    _check = _run_recurrence(torch.float32, 32, 40, (0.8,) * 5, [[2, 1]] * 4 + [[3]] * 200, [0, 1, 2, 3] + [-1] * 200, 3, False)
    got, want = _check[0], _check[1]
    for row in range(4):
        _near(got[row], want[row], torch.float32, f"row {row}")


@pytest.mark.parametrize("d, dv, heads", [(16, 16, 3), (64, 64, 5), (32, 40, 4), (48, 8, 2), (128, 80, 2), (96, 136, 2), (256, 24, 1)])
def test_recurrence_by_chunks_on_the_matrix_cores(d, dv, heads):
    """The same rows through the three launches over chunks: chunks that are full, that end early, rows of several chunks."""
    _check_recurrence(torch.bfloat16, d, dv, DECAYS[:heads], chunks=True)


def test_many_rows_of_chunks():
    """More rows than a wave looks at at a time when a workgroup finds its chunk."""
    counts = [1 + (i * 37) % 90 for i in range(140)]
    slots = [i if i < 5 else -1 for i in range(140)]
    got, want, _state, _states = _run_recurrence(torch.bfloat16, 32, 16, (0.9, 0.99), [[c] for c in counts], slots, 9, True)
    for row in range(140):
        if slots[row] >= 0:
            _near(got[row], want[row], torch.bfloat16, f"row {row}", atol=5e-2)
        else:
            assert float(got[row].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("dim", [4, 70, 320, 1000, 4096, 9000])
def test_gated_norm_of_whole_rows_kernel(dim, dtype):
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(dim)
    n = 5
    x = torch.randn(n, dim, generator=gen) * torch.tensor([1.0, 1e-3, 30.0, 0.0, 2.0])[:, None]
    gain = 1 + 0.3 * torch.randn(dim, generator=gen)
    gate = torch.randn(n, dim + 12, generator=gen).to(dtype)                       # columns of wider rows
    out = torch.full((n, dim), float("nan"), dtype=dtype, device=DEV)
    core.gated_rmsnorm(x.to(DEV), gain.to(DEV), 1e-4, gate.to(DEV)[:, 12:], out)
    want = plain.rms(x.double(), 1e-4) * gain.double() * torch.sigmoid(gate[:, 12:].double())
    _near(out, want, dtype, "gated", rtol=1e-2 if dtype == torch.bfloat16 else 1e-5, atol=1e-6)
    core.gated_rmsnorm(x.to(DEV), None, 1e-4, None, out)
    _near(out, plain.rms(x.double(), 1e-4), dtype, "neither gain nor gate", rtol=1e-2 if dtype == torch.bfloat16 else 1e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("dim", [4, 70, 300, 1024, 1500, 4096, 8192, 9000])
def test_a_normalised_sublayer_added_and_the_next_norm_kernel(dim, dtype):
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(dim)
    n = 3
    x, delta = torch.randn(n, dim, generator=gen) * 4, torch.randn(n, dim, generator=gen) * 0.01
    g1, g2 = 1 + 0.3 * torch.randn(dim, generator=gen), 1 + 0.3 * torch.randn(dim, generator=gen)
    want = x.double() + plain.rms(delta.double(), 1e-5) * g1.double()
    stream = x.to(DEV).clone()
    rows = torch.full((n, dim), float("nan"), dtype=dtype, device=DEV)
    core.add_normed(stream, delta.to(DEV), (g1.to(DEV), 1e-5), (g2.to(DEV), 1e-3), rows)
    _near(stream, want, torch.float32, "stream")
    _near(rows, plain.rms(want, 1e-3) * g2.double(), dtype, "rows", rtol=1e-2 if dtype == torch.bfloat16 else 1e-5, atol=1e-5)
    stream = x.to(DEV).clone()
    core.add_normed(stream, delta.to(DEV), (g1.to(DEV), 1e-5))
    _near(stream, want, torch.float32, "without a second norm")


def test_the_embedding_output_at_a_junction():
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(4)
    x, x0, vector = torch.randn(7, 33, generator=gen), torch.randn(7, 33, generator=gen), torch.randn(33, generator=gen)
    for dtype in DTYPES:
        got = x.to(DEV).clone()
        core.add_vector(got, vector.to(DEV, dtype), x0.to(DEV))
        _near(got, x.double() + x0.double() + vector.to(dtype).double(), torch.float32, "both")


@pytest.mark.parametrize("outputs, top", [(6, 2), (5, 5), (1, 1), (64, 8), (200, 6), (512, 4)])
def test_choice_by_logits_kernel(outputs, top):
    """The ``top`` largest logits and the softmax over those alone, where the others hold most of the mass of a softmax over
    all, and where logits lie so far apart that a score would underflow."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(outputs)
    n = 37
    logits = torch.randn(n, outputs + 1, generator=gen) * torch.tensor([1.0, 0.01, 60.0] * 13)[:n, None]
    chosen = torch.zeros(n, top, dtype=torch.int32, device=DEV)
    weights = torch.zeros(n, top, device=DEV)
    core.route(logits.to(DEV), outputs, None, top, 0, 0, 1.0, chosen, weights, weigh_chosen=True)
    order, want = plain.routing(logits[:, :outputs].double(), top)
    assert torch.equal(chosen.cpu().long(), order)
    _near(weights, want, torch.float32, "weights", atol=1e-6, rtol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("n, dim, ff, n_experts, top", [(3, 100, 36, 5, 2), (70, 128, 48, 6, 3), (200, 64, 96, 4, 1), (150, 192, 80, 33, 4), (90, 16, 176, 3, 2)])
def test_plain_experts_and_the_weighted_sum_kernels(n, dim, ff, n_experts, top, dtype):
    """Experts of two linears with the square of relu between, pair by pair and (bfloat16) listed by expert; the weighted
    sum with a gated shared expert, normalised, added into the stream and followed by the next norm."""
    from kestrel_amd.engine.batch import Workspace
    from kestrel_amd.ops import core, fast
    from kestrel_amd.ops.linear import activation_code

    gen = torch.Generator().manual_seed(n + dim)
    h = torch.randn(n, dim, generator=gen).to(dtype)
    up = (torch.randn(n_experts, ff, dim, generator=gen) / math.sqrt(dim)).to(dtype)
    down = (torch.randn(n_experts, dim, ff, generator=gen) / math.sqrt(ff)).to(dtype)
    chosen = torch.stack([torch.randperm(n_experts, generator=gen)[:top] for _ in range(n)]).to(torch.int32)
    weights = torch.rand(n, top, generator=gen)
    shared, sg = torch.randn(n, dim, generator=gen), torch.randn(n, generator=gen)
    w = {}
    for e in range(n_experts):
        w[f"e{e}.up"], w[f"e{e}.down"] = up[e].double(), down[e].double()
    want = torch.stack([sum(float(weights[t, k]) * plain.expert(h[t:t + 1].double(), w, f"e{int(chosen[t, k])}")[0] for k in range(top))
                        for t in range(n)]) + torch.sigmoid(sg.double())[:, None] * shared.double()
    act = activation_code("relu_squared")
    flat = chosen.to(DEV).view(-1)
    hidden = torch.zeros(n * top, ff, dtype=dtype, device=DEV)
    y = torch.full((n * top, dim), float("nan"), device=DEV)
    core.experts_linear(h.to(DEV), top, up.to(DEV), flat, hidden, act)
    core.experts_linear(hidden, 1, down.to(DEV), flat, y)
    gate_column = torch.stack([torch.zeros(n), sg], dim=1).to(DEV)[:, 1]          # a column with a stride
    g1, g2 = 1 + 0.2 * torch.randn(dim, generator=gen), 1 + 0.2 * torch.randn(dim, generator=gen)
    x = torch.randn(n, dim, generator=gen) * 2
    stream = x.double() + plain.rms(want, 1e-5) * g1.double()

    def combined(pairs, what):
        got = torch.zeros(n, dim, device=DEV)
        core.experts_combine(pairs, h.to(DEV), chosen.to(DEV), weights.to(DEV), n_experts, shared.to(DEV), gate_column, got, False)
        _near(got, want, dtype, what, atol=2e-5 if dtype == torch.float32 else 3e-2)
        got = x.to(DEV).clone()
        rows = torch.full((n, dim), float("nan"), dtype=dtype, device=DEV)
        core.experts_combine_normed(pairs, h.to(DEV), chosen.to(DEV), weights.to(DEV), n_experts, shared.to(DEV), gate_column, got,
                                    (g1.to(DEV), 1e-5), (g2.to(DEV), 1e-5), rows)
        _near(got, stream, dtype, what + ", normed", atol=2e-5 if dtype == torch.float32 else 4e-2)
        _near(rows, plain.rms(stream, 1e-5) * g2.double(), dtype, what + ", the next norm", atol=3e-5 if dtype == torch.float32 else 4e-2)

    combined(y, "pair by pair")
    if dtype == torch.bfloat16 and dim % 16 == 0 and ff % 16 == 0:
        y = torch.full((n * top, dim), float("nan"), device=DEV)
        assert fast.experts_feed_forward_bf16(h.to(DEV), up.to(DEV), down.to(DEV), chosen.to(DEV), None, y, act, Workspace(torch.device(DEV)))
        combined(y, "by expert")
    if dtype == torch.bfloat16 and dim % 8 == 0 and ff % 8 == 0 and n * top <= 512:
        y = torch.full((n * top, dim), float("nan"), device=DEV)
        assert fast.experts_few_bf16(h.to(DEV), up.to(DEV), down.to(DEV), chosen.to(DEV), torch.zeros(n * top, ff, dtype=dtype, device=DEV), y, act)
        combined(y, "few pairs")


@pytest.mark.parametrize("kernel, dtype", [("generic", torch.float32), ("generic", torch.bfloat16), ("mfma", torch.bfloat16)],
                         ids=["generic-fp32", "generic-bf16", "mfma-bf16"])
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("rank, heads, window", [(64, 4, 24), (48, 40, 7), (128, 3, 33), (192, 2, 64), (32, 1, 1), (80, 5, None)])
def test_windowed_latents_and_a_gate_per_head(rank, heads, window, cut, kernel, dtype):
    """Queries over cached latents behind a window, one of whose keys stands out for every query: the last one inside the
    window for some queries, the first one outside for others (it would take nearly all the weight); pages behind the
    window are given back and hold NaN; one gate number per head, some nearly shut."""
    from kestrel_amd.ops import core, fast

    lengths, starts = CUTS[cut]
    case = PackedStep(lengths, starts, window, 0, seed=rank + heads)
    scale = 1.0 / math.sqrt(rank)
    rows, q = [], []
    for n, s in zip(lengths, starts):
        c = torch.randn(n, 1, rank, generator=case.gen)
        queries = torch.randn(n - s, heads, rank, generator=case.gen)
        if window is not None:
            # every query of the row leans towards one direction; every (window)th key lies along it
            lean = torch.randn(rank, generator=case.gen)
            lean = lean / lean.norm() * math.sqrt(rank)
            c[n % window::window, 0] = lean
            queries = queries * 0.2 + lean * (8.0 / math.sqrt(rank))
        rows.append(c.to(dtype))
        q.append(queries.to(dtype))
    gate = (torch.randn(case.n, heads + 3, generator=case.gen) * 3).to(dtype)
    out = torch.full((case.n, heads * rank), float("nan"), dtype=dtype, device=DEV)
    packed_q, pages, gates = torch.cat(q).reshape(case.n, -1).to(DEV), case.pages(rows), gate.to(DEV)[:, 3:]
    if kernel == "mfma":
        assert fast.attention_latent_bf16(packed_q, pages, case.table, case.token_row, case.kv_hi, out, scale, heads, rank, rank, None,
                                          case.batch, kv_lo=case.kv_lo, head_gate=gates)
    else:
        core.attention_generic(packed_q, pages, None, case.table, case.token_row, case.kv_lo, case.kv_hi, out, scale, heads, 1, rank, rank,
                               values_in_keys=True, gate=gates, gate_per_head=True)
    want = []
    for r, (n, s) in enumerate(zip(lengths, starts)):
        c = rows[r].double()[:, 0]
        seen = plain.window_mask(n, window)[s:]
        want.append(torch.stack([plain.softmax_over((q[r].double()[:, h] @ c.T) * scale, seen) @ c for h in range(heads)], dim=1))
    want = torch.cat(want) * torch.sigmoid(gate[:, 3:].double())[:, :, None]
    _near(out.view(case.n, heads, rank), want, dtype, "latents")


@pytest.mark.parametrize("host_knows", [True, False], ids=["launched", "captured"])
@pytest.mark.parametrize("lengths, starts", [([70, 300, 9, 101, 64, 200, 129], [0, 100, 7, 100, 0, 137, 0]), ([500], [300]), ([40, 64], [0, 1])],
                         ids=["mixed", "one portion", "none long enough"])
@pytest.mark.parametrize("rank, heads, d, dv, window", [(64, 4, 32, 24, 24), (48, 2, 64, 64, 7), (144, 3, 32, 80, 33), (128, 1, 128, 128, 64), (80, 6, 48, 4, 200)])
def test_latents_lifted_for_long_portions(rank, heads, d, dv, window, lengths, starts, host_knows):
    """The mixer's core on a step whose long portions are lifted to keys and values per head while its short portions and
    single tokens stay with the latents; one key stands out at the window's edge; pages given back hold NaN. ``captured``: the
    host does not know what the step brings (as when it was captured), both halves are launched."""
    from kestrel_amd.engine.batch import GroupBatch
    from kestrel_amd.parts.base import LayerCache
    from kestrel_amd.parts.latent_attention import LatentAttention
    from kestrel_amd.parts.specs import LatentAttentionSpec, PositionSpec

    bf = torch.bfloat16
    case = PackedStep(lengths, starts, window, 0, seed=rank + d)
    gen = case.gen
    scale = 1.0 / math.sqrt(d)
    mixer = LatentAttention(LatentAttentionSpec("latent_attention", 32, heads, d, 0, dv, None, rank, scale, 1e-5, PositionSpec("none"),
                                                head_sinks=False, gate_per_head=True, window=window))
    w = {name: (torch.randn(spec.shape, generator=gen) * 0.2).to(bf) for name, spec in mixer.params().items()}
    mixer.bind({k: v.to(DEV) for k, v in w.items()}, bf, torch.device(DEV))
    assert mixer.lift_weight is not None
    uk, uv = w["uk.weight"].double(), w["uv.weight"].double()
    rows, q = [], []
    for n, s in zip(lengths, starts):
        c = torch.randn(n, 1, rank, generator=gen)
        lean = torch.randn(rank, generator=gen)
        lean = lean / lean.norm() * math.sqrt(rank)
        c[n % window::window, 0] = lean
        key = (uk @ lean.double()).reshape(heads, d)
        queries = 0.2 * torch.randn(n - s, heads, d, generator=gen).double() + key * (9.0 / (scale * key.pow(2).sum(dim=1, keepdim=True)))
        rows.append(c.to(bf))
        q.append(queries.float().to(bf))
    down = torch.zeros(case.n, mixer.down_dim, dtype=bf)
    down[:, :heads * d] = torch.cat(q).reshape(case.n, -1)
    gate = (torch.randn(case.n, heads, generator=gen) * 3).to(bf)
    down[:, heads * d + rank:heads * d + rank + heads] = gate
    batch = case.batch
    batch.n_tokens, batch.n_rows, batch.token_row, batch.kv_hi = case.n, len(lengths), case.token_row, case.kv_hi
    batch.kv_len, batch.positions = _i32(lengths), _i32([0] * case.n)
    batch.host = {"q_lens": [n - s for n, s in zip(lengths, starts)] if host_knows else []}
    pages = case.pages(rows)
    batch.groups = {0: GroupBatch(block_table=case.table, slots=_i32([-1] * case.n), kv_lo=case.kv_lo, page_size=16)}
    got = mixer.attend(down.to(DEV), batch, LayerCache(group=0, tensors={"k": pages}))
    want = []
    for r, (n, s) in enumerate(zip(lengths, starts)):
        c = rows[r].double()[:, 0]
        k, v = (c @ uk.T).reshape(n, heads, d), (c @ uv.T).reshape(n, heads, dv)
        seen = plain.window_mask(n, window)[s:]
        want.append(torch.stack([plain.softmax_over((q[r].double()[:, h] @ k[:, h].T) * scale, seen) @ v[:, h] for h in range(heads)], dim=1))
    want = torch.cat(want) * torch.sigmoid(gate.double())[:, :, None]
    spread = float(want.std())
    _near(got.view(case.n, heads, dv), want, bf, "heads", atol=3e-2 * max(1.0, 2 * spread), rtol=2e-2)


def test_latents_made_ready_without_a_rotated_part():
    """Only the latent is normalised and cached: rows of ``[q | latent | gate]`` with no latent of queries and no shared part."""
    from kestrel_amd.ops import core

    gen = torch.Generator().manual_seed(12)
    n, q, rank, ps = 5, 24, 40, 4
    for dtype in DTYPES:
        down = (torch.randn(n, q + rank + 3, generator=gen) * 2).to(dtype)
        gain = 1 + 0.3 * torch.randn(rank, generator=gen)
        slots = [3, 4, 5, -1, 12]
        cache = torch.zeros(4, 1, ps, rank, dtype=dtype, device=DEV)
        core.latent_prepare(down.to(DEV), 0, 0, None, None, q, rank, gain.to(DEV), 0, None, "halves", _i32(list(range(n))), _i32(slots), cache, 1e-4)
        want = plain.rms(down[:, q:q + rank].double(), 1e-4) * gain.double()
        got = cache.cpu().reshape(-1, rank)
        for t, slot in enumerate(slots):
            if slot >= 0:
                _near(got[slot], want[t], dtype, f"token {t}", rtol=1e-2 if dtype == torch.bfloat16 else 2e-5)
        assert float(got[[0, 1, 2, 6, 7, 8, 9, 10, 11, 13, 14, 15]].abs().max()) == 0.0


@pytest.mark.parametrize("rows, columns", [(1, 40), (9, 40), (70, 1024), (255, 1024), (256, 1024), (300, 1048), (300, 1020)])
def test_relu_squared_in_every_linear_kernel(rows, columns):
    """In the epilogue of this package's kernels, and as a pass over the vendor library's product for large outputs; columns
    behind the output's in its buffer are left alone."""
    from kestrel_amd.ops.linear import activation_code, linear

    gen = torch.Generator().manual_seed(rows)
    a, w = torch.randn(rows, 64, generator=gen).bfloat16(), (torch.randn(columns, 64, generator=gen) * 0.2).bfloat16()
    buffer = torch.full((rows, columns + 8), 7.0, dtype=torch.bfloat16, device=DEV)
    linear(a.to(DEV), w.to(DEV), None, buffer[:, :columns], act=activation_code("relu_squared"))
    _near(buffer[:, :columns], plain.relu_squared(a.double() @ w.double().T), torch.bfloat16, "relu squared", atol=1e-4)
    assert bool((buffer[:, columns:] == 7.0).all())


def test_the_matrix_core_kernels_run_where_sizes_allow():
    """In bfloat16 the models whose sizes the matrix-core kernels take run them for prompts, and the model of odd sizes the
    generic ones where they do not fit."""
    from kestrel_amd.ops import fast

    calls = {}
    names = ("attention_biased_bf16", "linear_attention_chunks_bf16", "experts_feed_forward_bf16", "heads_linear_bf16", "latent_expand_bf16")
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
            for length in (50, 270):             # (too short for its latents to be lifted and for lists of experts, and long enough)
                helpers.replay(_runner(folder, torch.bfloat16), {"r": Request("r", _ids(folder, 900, length))}, [[("r", length)]])
            assert set(calls) == set(names) and all(bool(d) for done in calls.values() for d in done), (model, calls)
    finally:
        for name in names:
            setattr(fast, name, originals[name])


# ================================================================================================ the model, cut every way
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("name", NAMES)
def test_every_layer(name, dtype):
    """The residual stream after every layer, then the logits."""
    from kestrel_amd.parts.block import Block

    folder = cases.folder_for(name, dtype)
    runner = _runner(folder, dtype)
    ids = _ids(folder, 1, 45)
    seen = []
    original = Block.forward

    def spy(self, x, *args, **kwargs):
        result = original(self, x, *args, **kwargs)
        seen.append(x.detach().double().cpu())
        return result

    Block.forward = spy
    try:
        got = helpers.replay(runner, {"r": Request("r", ids)}, [[("r", len(ids))]])
    finally:
        Block.forward = original
    streams = []
    want = plain.forward(cases.config_of(folder), cases.stored_weights(folder), ids, streams)
    assert len(seen) == len(streams)
    for layer, (a, b) in enumerate(zip(seen, streams)):
        rms = ((a - b).pow(2).mean(dim=-1) / b.pow(2).mean(dim=-1)).sqrt()
        assert float(rms.max()) <= (2e-5 if dtype == torch.float32 else 3e-2), f"{name} layer run {layer}: {float(rms.max()):.3g}"
    _close(got["r"], want, dtype, f"{name} logits")


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
    """Steps replayed as graphs, one graph serving steps of different make-up in turn: long portions (whose latents are
    lifted) alone, beside short ones and single tokens, and steps of the same number of tokens without a long one; in
    pages that were given back and hold NaN."""
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
            bound = torch.clamp(_what_rounding_does(folder, req.ids)[places], min=0.04)
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
    """On a folder crafted so that it shows (``cases.crafted``; ``test_vufolorn_cpu.py`` measures by how much): a token that
    calls and, at a chosen distance before it, the token it calls for: just inside and just outside either window, at a
    page's border, far back, and at the sequence's first place; inside a prompt, decoded alone, and with all but two tokens
    decoded."""
    base = cases.folder_for("P", dtype)
    folder = cases.crafted(base)
    windows = [layer["mixer"]["mask"]["size"] for layer in cases.config_of(base)["layers"] if "mask" in layer["mixer"]]
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
            _close(got["r"], want, dtype, f"distance {distance}, prompt of {head}")


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
