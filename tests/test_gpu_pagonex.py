"""Pagonex on the GPU against the plain implementation (tests/plain_pagonex.py): every mechanism alone, then
the engine under every way of cutting requests into steps."""
import functools
import json
import math
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_pagonex as P
from tiny_pagonex import CONFIGS, SEEDS, STD_BY_SUFFIX, config

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}

# Float arithmetic against the plain model in double.  Whatever the design adds shows at 5e-3 and more when left
# out (test_what_the_design_adds_would_show_if_left_out).
FLOAT_KERNEL = 2e-5           # a row out of one kernel
FLOAT_STATE = 1e-4            # a row of the recurrence's output, and its state
FLOAT_LOGITS = 3e-4           # a row of logits, a layer's sum
FLOAT_SAME = 3e-5             # the same logits by another cut or in another batch
BF16_KERNEL = 8e-3            # a row out of one kernel that rounds its result to bfloat16


def _rel_rows(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    got, want = got.double().cpu(), want.double().cpu()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-30)


def _rel_rms(got: torch.Tensor, want: torch.Tensor) -> float:
    """The largest error of a row, as rms(difference) / rms(row)."""
    return float(_rel_rows(got, want).max())


def _within_noise(err: torch.Tensor, noise: torch.Tensor, what: str) -> None:
    """`err`: per row, the engine's bfloat16 error; `noise`: per row, how far the plain model moves when it rounds to
    bfloat16 every tensor that a 16-bit engine may keep in 16 bits, and nothing of what the design computes in 32 bits.
    A row's limit is three times its noise (at least three times the median row's); at most three rows in a
    hundred (or one) may exceed it, none two and a half times it.  The float32 runs of the same tests are the sharp ones."""
    limit = 3.0 * torch.maximum(noise, noise.median())
    over, far = int((err > limit).sum()), int((err > 2.5 * limit).sum())
    worst = int((err / limit).argmax())
    assert over <= max(1, 0.03 * err.numel()) and far == 0, \
        f"{what}: {over} of {err.numel()} rows over their limit, {far} far over; row {worst}: {float(err[worst]):.2e} (limit {float(limit[worst]):.2e})"


def _dithered(k):
    """bfloat16 rounding on a grid shifted by k / 1024 of a value: another draw of the same rounding noise."""
    f = 1.0 + k * 2.0 ** -10
    return lambda x: P.store_bf16(x * f) / f


def _noise_rows(run):
    """Per row, how far rounding alone moves a result: the largest of three draws, and of the two neighbouring rows."""
    exact = run(P._same)
    outs = [run(P.store_bf16), run(_dithered(1)), run(_dithered(-1))]
    many = isinstance(exact, list)
    per = []
    for i in range(len(exact) if many else 1):
        w = exact[i] if many else exact
        n = torch.stack([_rel_rows(o[i] if many else o, w) for o in outs]).max(0).values
        pad = torch.cat([n[:1], n, n[-1:]])
        per.append(torch.stack([pad[:-2], pad[1:-1], pad[2:]]).max(0).values)
    return (exact, per) if many else (exact, per[0])


class _Step:
    """What the kernels read of a step."""

    def __init__(self, lens, starts, slots, ids=None):
        from sharpinference_amd import ops

        self.n_entries, self.n_tokens, self.max_entry_len = len(lens), sum(lens), max(lens)
        cu = [0]
        for n in lens:
            cu.append(cu[-1] + n)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
        self.cu_tokens = i32(cu)
        self.entry_of_token = i32([e for e, n in enumerate(lens) for _ in range(n)])
        self.positions = i32([s + i for s, n in zip(starts, lens) for i in range(n)])
        self.state_slots = i32(slots)
        self.token_ids = i32(ids) if ids is not None else None
        chunks, ents = ops.delta_chunks_of(lens, cu)
        self.lists = (i32(chunks.reshape(-1)), i32(ents.reshape(-1)))
        self.single = max(lens) == 1


# steps of three requests: one token, a few, many; two entries of one token each; a request left out of a step; pairs
# and singles at the end
PLAN = [[("a", 1), ("b", 40)], [("b", 1), ("c", 7), ("a", 2)], [("c", 1), ("a", 1)], [("a", 9), ("c", 1)], [("c", 1), ("a", 2), ("b", 1)],
        [("b", 1)], [("a", 1), ("b", 1), ("c", 1)], [("a", 1), ("b", 33), ("c", 16)], [("b", 1), ("a", 1)]]
TOTAL = {r: sum(n for step in PLAN for q, n in step if q == r) for r in "abc"}
SLOT_OF = {"a": 3, "b": 0, "c": 1}


def _over_plan(rows_of, call):
    """Runs `call(rows, ctx)` over PLAN, returns each request's outputs in order."""
    got = {r: [] for r in TOTAL}
    at = {r: 0 for r in TOTAL}
    for step in PLAN:
        ctx = _Step([n for _, n in step], [at[r] for r, _ in step], [SLOT_OF[r] for r, _ in step])
        take = lambda x: torch.cat([x[r][at[r]:at[r] + n] for r, n in step]).to(DEV)
        o = call([take(x) for x in rows_of] if isinstance(rows_of, list) else take(rows_of), ctx)
        i = 0
        for r, n in step:
            got[r].append(o[i:i + n].cpu())
            i += n
            at[r] += n
    return {r: torch.cat(v) for r, v in got.items()}


# ---------------------------------------------------------------------------
# the delta rule alone
# ---------------------------------------------------------------------------
def _delta_case(H, G, dk, dv, taps, dtype, seed, decay_scale=1.0):
    g = torch.Generator().manual_seed(seed)
    C = 2 * G * dk + H * dv
    rows = {r: torch.randn(n, C + 11, generator=g).to(DT[dtype]) for r, n in TOTAL.items()}      # eleven columns that belong to nobody
    ld = {r: -torch.exp(torch.randn(n, H * dk, generator=g) * 2.0 - 2.0) * decay_scale for r, n in TOTAL.items()}
    beta = {r: torch.randn(n, H + 3, generator=g) * 2.0 for r, n in TOTAL.items()}
    gate = {r: torch.randn(n, H * dv, generator=g).to(DT[dtype]) for r, n in TOTAL.items()}
    conv_w = torch.randn(C, taps, generator=g) * 0.7
    norm_w = 0.5 + torch.rand(dv, generator=g)
    return rows, ld, beta, gate, conv_w, norm_w


def _plain_delta(rows, ld, beta, gate, conv_w, norm_w, H, G, dk, dv, eps, c_off=0, beta_off=0):
    T = rows.shape[0]
    u = rows.double()[:, c_off:c_off + 2 * G * dk + H * dv]
    u = P.silu(P.causal_conv(u, conv_w.double()))
    q = P.unit_vector(u[:, :G * dk].reshape(T, G, dk)) * dk ** -0.5
    k = P.unit_vector(u[:, G * dk:2 * G * dk].reshape(T, G, dk))
    v = u[:, 2 * G * dk:].reshape(T, H, dv)
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    o, S = P.delta_rule(q, k, v, torch.exp(ld.double()).reshape(T, H, dk), torch.sigmoid(beta.double()[:, beta_off:beta_off + H]))
    y = P.rms_norm(o, norm_w.double(), eps) * torch.sigmoid(gate.double()).reshape(T, H, dv)
    return y.reshape(T, -1), o.reshape(T, -1), S


def _run_delta(ops, x, ld, beta, gate, ctx, conv_w, ring, state, norm_w, H, G, dk, dv, eps, c_off=0, beta_off=0, chunked=None):
    args = (x, c_off, conv_w, ring, ld, beta, beta_off, state, ctx, H, G, dk, dv)
    if ctx.single and not chunked:
        return ops.delta_step(*args, norm_w, eps, gate)
    o = ops.delta_chunks(*args, ctx.lists)
    return ops.group_norm_gate(o, norm_w.repeat(H).contiguous(), eps, H, x.dtype, gate, 0, ops.GATE_SIGMOID_ACT)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, G, dk, dv, taps", [(2, 1, 10, 24, 3), (6, 2, 20, 12, 2), (3, 3, 32, 16, 1), (4, 2, 64, 50, 4), (1, 1, 136, 40, 8),
                                                (2, 2, 128, 128, 4), (2, 1, 256, 9, 5), (3, 1, 72, 200, 3), (1, 1, 1, 1, 2), (5, 5, 33, 17, 6)])
def test_the_delta_rule_moves_every_entry_from_its_slots_state(dtype, H, G, dk, dv, taps):
    """Convolution, unit vectors, decays from almost none to complete, corrections, head norm and gate, in both forms, over
    steps of every kind, against the plain recurrence over whole sequences; states and rings in slots 3, 0 and 1 of five."""
    from sharpinference_amd import ops

    eps = 1e-5
    rows, ld, beta, gate, conv_w, norm_w = _delta_case(H, G, dk, dv, taps, dtype, dk + dv)
    C = conv_w.shape[0]
    state = torch.zeros(5, *ops.delta_state_shape(H, dk, dv), device=DEV)
    ring = torch.zeros(5, taps, C, device=DEV) if taps > 1 else None
    for t in (state, ring):
        if t is not None:
            t[2].fill_(9.0)                                      # a slot no entry names
    cw, nw = conv_w.to(DEV), norm_w.to(DEV)
    call = lambda xs, ctx: _run_delta(ops, *xs, ctx, cw, ring, state, nw, H, G, dk, dv, eps, c_off=7, beta_off=2)
    got = _over_plan([rows, ld, beta, gate], call)
    for r in TOTAL:
        want, _, S = _plain_delta(rows[r].float(), ld[r], beta[r], gate[r].float(), conv_w, norm_w, H, G, dk, dv, eps, 7, 2)
        heads = lambda y: y.reshape(-1, dv)
        assert _rel_rms(heads(got[r]), heads(want)) < (FLOAT_STATE if dtype == "float32" else BF16_KERNEL), r
        kept = ops.delta_state_matrices(state[SLOT_OF[r]], dk, dv)
        assert _rel_rms(kept.reshape(H, -1), S.reshape(H, -1)) < FLOAT_STATE, r
        for back in range(min(taps, TOTAL[r]) if taps > 1 else 0):
            p = TOTAL[r] - 1 - back
            if back < taps - 1:
                assert torch.equal(ring[SLOT_OF[r], p % taps].cpu(), rows[r][p, 7:7 + C].float()), (r, back)
    assert bool((state[2] == 9.0).all()) and not bool(state[4].any())
    assert ring is None or (bool((ring[2] == 9.0).all()) and not bool(ring[4].any()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_two_forms_of_the_delta_rule_give_the_same(dtype):
    """Single tokens through the chunked form: the same outputs and states to rounding."""
    from sharpinference_amd import ops

    H, G, dk, dv, taps, eps = 4, 2, 24, 40, 3, 1e-6
    rows, ld, beta, gate, conv_w, norm_w = _delta_case(H, G, dk, dv, taps, dtype, 5)
    outs = []
    for chunked in (False, True):
        state = torch.zeros(5, *ops.delta_state_shape(H, dk, dv), device=DEV)
        ring = torch.zeros(5, taps, conv_w.shape[0], device=DEV)
        call = lambda xs, ctx: _run_delta(ops, *xs, ctx, conv_w.to(DEV), ring, state, norm_w.to(DEV), H, G, dk, dv, eps, chunked=chunked)
        outs.append((_over_plan([rows, ld, beta, gate], call), state.cpu(), ring.cpu()))
    for r in TOTAL:
        assert _rel_rms(outs[0][0][r], outs[1][0][r]) < (FLOAT_SAME if dtype == "float32" else BF16_KERNEL)
    assert _rel_rms(outs[0][1].reshape(5, -1)[[0, 1, 3]], outs[1][1].reshape(5, -1)[[0, 1, 3]]) < FLOAT_SAME
    assert torch.equal(outs[0][2], outs[1][2])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [[640], [600, 39, 1], [16] * 40, [39, 2, 599], [40] + [1] * 600])
def test_one_token_far_back_is_still_in_the_state(dtype, cuts):
    """A key 600 tokens back in a direction of its own that the last query points at, decays of almost 1 in head 0 and
    strong ones in head 1: head 0 reads the value that was stored then, head 1 has forgotten it."""
    from sharpinference_amd import ops

    H, G, dk, dv, T, eps = 2, 2, 32, 16, 640, 1e-6
    g = torch.Generator().manual_seed(5)
    rows = torch.randn(T, 2 * G * dk + H * dv, generator=g)
    for h in range(2):
        rows[:, h * dk] = 0.0                                    # nobody's query or key has anything in channel 0 ...
        rows[:, G * dk + h * dk] = 0.0
        rows[39, G * dk + h * dk: G * dk + (h + 1) * dk] = 0.0
        rows[39, G * dk + h * dk] = 5.0                          # ... but this key
        rows[T - 1, h * dk:(h + 1) * dk] = 0.0
        rows[T - 1, h * dk] = 5.0                                # ... and the last query
    rows = rows.to(DT[dtype])
    ld = torch.full((T, H * dk), -1e-4)
    ld[:, dk:] = -0.05
    beta, gate = torch.full((T, H), 3.0), torch.zeros(T, H * dv).to(DT[dtype])
    conv_w, norm_w = torch.ones(rows.shape[1], 1), torch.ones(dv)
    state = torch.zeros(2, *ops.delta_state_shape(H, dk, dv), device=DEV)
    o, at = [], 0
    for n in cuts:
        ctx = _Step([n], [at], [1])
        o.append(_run_delta(ops, rows[at:at + n].to(DEV), ld[at:at + n].to(DEV), beta[at:at + n].to(DEV), gate[at:at + n].to(DEV), ctx,
                            conv_w.to(DEV), None, state, norm_w.to(DEV), H, G, dk, dv, eps).cpu())
        at += n
    got = torch.cat(o)
    want, raw, _ = _plain_delta(rows.float(), ld, beta, gate.float(), conv_w, norm_w, H, G, dk, dv, eps)
    stored = P.silu(rows[39, 2 * G * dk:2 * G * dk + dv].double())
    assert _rel_rms(raw[T - 1:, :dv] / raw[T - 1, :dv].norm(), (stored / stored.norm())[None]) < 1e-3
    assert float(raw[T - 1, dv:].norm()) < 1e-6 * float(raw[T - 1, :dv].norm())
    assert _rel_rms(got[T - 1:, :dv], want[T - 1:, :dv]) < (FLOAT_STATE if dtype == "float32" else BF16_KERNEL)


@pytest.mark.parametrize("scale", [0.0, 60.0, 1e4])
def test_decays_from_none_to_complete(scale):
    """No decay at all, channels forgotten within a token, and logarithms far below what an exponential holds: finite
    and right (every exponent of the chunked form is at most zero)."""
    from sharpinference_amd import ops

    H, G, dk, dv, taps, eps = 2, 1, 40, 24, 3, 1e-5
    rows, ld, beta, gate, conv_w, norm_w = _delta_case(H, G, dk, dv, taps, "float32", 9, decay_scale=scale)
    state = torch.zeros(5, *ops.delta_state_shape(H, dk, dv), device=DEV)
    ring = torch.zeros(5, taps, conv_w.shape[0], device=DEV)
    call = lambda xs, ctx: _run_delta(ops, *xs, ctx, conv_w.to(DEV), ring, state, norm_w.to(DEV), H, G, dk, dv, eps)
    got = _over_plan([rows, ld, beta, gate], call)
    for r in TOTAL:
        want, _, _ = _plain_delta(rows[r], ld[r], beta[r], gate[r], conv_w, norm_w, H, G, dk, dv, eps)
        assert torch.isfinite(got[r]).all() and _rel_rms(got[r], want) < FLOAT_STATE


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T, rank, H, dk, rank1, N1", [(1, 7, 3, 5, 9, 11), (70, 24, 2, 40, 16, 64), (130, 128, 4, 64, 33, 100), (16, 1, 1, 1, 3, 1)])
def test_products_through_a_narrow_middle_and_the_decays_logarithms(dtype, T, rank, H, dk, rank1, N1):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(T + rank)
    x = torch.randn(T, rank + rank1 + 5, generator=g)
    w, w1 = (torch.randn(n, r, generator=g).to(DT[dtype]) for n, r in ((H * dk, rank), (N1, rank1)))
    bias, a_log = torch.randn(H * dk, generator=g) * 4.0, torch.randn(H, generator=g) * 2.0
    ld, z = ops.lowrank(x.to(DEV), (2, w.to(DEV), bias.to(DEV), a_log.to(DEV)), (2 + rank, w1.to(DEV)))
    logit = x.double()[:, 2:2 + rank] @ w.double().T + bias.double()
    want = -torch.exp(a_log.double()).repeat_interleave(dk)[None] * P.softplus(logit)
    assert ld.dtype == torch.float32 and _rel_rms(ld, want) < FLOAT_KERNEL
    assert z.dtype == DT[dtype]
    want1 = x.double()[:, 2 + rank:2 + rank + rank1] @ w1.double().T
    assert (z.double().cpu() - want1).norm() / want1.norm() < (FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL)
    alone, none = ops.lowrank(x.to(DEV), (2, w.to(DEV), bias.to(DEV), a_log.to(DEV)))
    assert none is None and torch.equal(alone, ld)


# ---------------------------------------------------------------------------
# norms, convolutions over the sum, the embedding
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W, T", [(64, 5), (77, 9), (1000, 3), (2048, 2), (9000, 2), (3, 4)])
def test_the_layer_norm_behind_a_branch_and_what_it_hands_on(dtype, W, T):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(W)
    h, y = torch.randn(T, W, generator=g), (torch.randn(T, W, generator=g) * 2.0 + 3.0).to(DT[dtype])
    w, b, w2, b2 = (torch.randn(W, generator=g) for _ in range(4))
    eps, eps2 = 1e-3, 1e-5
    new = h.double() + P.layer_norm(y.double(), w.double(), b.double(), eps)
    tol = FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL
    d = lambda x: x.to(DEV)
    hd = d(h).clone()
    act = ops.layer_norm(hd, d(y), d(w), d(b), eps, out_dtype=DT[dtype])
    assert _rel_rms(hd, new) < FLOAT_KERNEL and torch.equal(act.cpu(), hd.cpu().to(DT[dtype]))
    hd = d(h).clone()
    assert ops.layer_norm(hd, d(y), d(w), d(b), eps) is None and _rel_rms(hd, new) < FLOAT_KERNEL
    # a second norm of the new sum; for some rows only (the sum then stays), with and without a branch waiting
    want = P.layer_norm(new, w2.double(), b2.double(), eps2)
    hd = d(h).clone()
    assert _rel_rms(ops.layer_norm(hd, d(y), d(w), d(b), eps, out_dtype=DT[dtype], norm=(d(w2), d(b2), eps2)), want) < tol
    rows = torch.tensor([T - 1, 0, 0], dtype=torch.int32, device=DEV)
    hd = d(h).clone()
    got = ops.layer_norm(hd, d(y), d(w), d(b), eps, rows=rows, out_dtype=DT[dtype], norm=(d(w2), d(b2), eps2))
    assert _rel_rms(got, want[[T - 1, 0, 0]]) < tol and torch.equal(hd.cpu(), h)
    got = ops.layer_norm(hd, rows=rows, out_dtype=DT[dtype], norm=(d(w2), d(b2), eps2))
    assert _rel_rms(got, P.layer_norm(h.double(), w2.double(), b2.double(), eps2)[[T - 1, 0, 0]]) < tol


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W", [64, 50])
def test_the_layer_norm_forms_a_weighted_sum_of_expert_rows_and_a_shared_row(dtype, W):
    from sharpinference_amd import ops

    T, k = 9, 3
    g = torch.Generator().manual_seed(W)
    ys, shared = torch.randn(T * k, W, generator=g).to(DT[dtype]), torch.randn(T, W, generator=g).to(DT[dtype])
    pos = torch.randperm(T * k, generator=g).to(torch.int32)
    wts = torch.rand(T, k, generator=g)
    h, w, b = torch.randn(T, W, generator=g), torch.randn(W, generator=g), torch.randn(W, generator=g)
    for sh in (shared, None):
        total = (ys.double()[pos.long()].reshape(T, k, W) * wts.double()[..., None]).sum(1) + (0 if sh is None else sh.double())
        hd = h.to(DEV)
        lazy = ops.ExpertSum(ys.to(DEV), pos.to(DEV), None if sh is None else sh.to(DEV), T, k, wts.to(DEV))
        ops.layer_norm(hd, lazy, w.to(DEV), b.to(DEV), 1e-5)
        assert _rel_rms(hd, h.double() + P.layer_norm(total, w.double(), b.double(), 1e-5)) < FLOAT_KERNEL


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W, taps", [(64, 4), (77, 3), (520, 2), (40, 8), (33, 1), (16, 5), (2056, 4)])
def test_the_convolution_over_the_sum_carries_its_inputs_from_step_to_step(dtype, W, taps):
    """x + conv(x) over steps of every kind (single tokens: inside the norm's kernel, with a branch folded in and without), the
    inputs before a step from the request's ring, zeros before the first token."""
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(W + taps)
    hs = {r: torch.randn(n, W, generator=g) for r, n in TOTAL.items()}
    ys = {r: torch.randn(n, W, generator=g).to(DT[dtype]) for r, n in TOTAL.items()}
    w, b, cw = torch.randn(W, generator=g), torch.randn(W, generator=g), torch.randn(W, taps, generator=g)
    for with_branch in (True, False):
        ring = torch.zeros(5, taps, W, device=DEV) if taps > 1 else None
        if ring is not None:
            ring[2].fill_(9.0)

        def call(xs, ctx):
            h, y = xs
            delta = (y, w.to(DEV), b.to(DEV)) if with_branch else (None, None, None)
            if ctx.single:
                return ops.layer_norm(h, *delta, 1e-5, out_dtype=DT[dtype], conv=(cw.to(DEV), ring, ctx))
            if with_branch:
                ops.layer_norm(h, *delta, 1e-5)
            return ops.residual_conv(h, cw.to(DEV), ring, ctx, DT[dtype])

        got = _over_plan([hs, ys], call)
        for r in TOTAL:
            x = hs[r].double() + (P.layer_norm(ys[r].double(), w.double(), b.double(), 1e-5) if with_branch else 0)
            assert _rel_rms(got[r], x + P.causal_conv(x, cw.double())) < (FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL), r
        assert ring is None or (bool((ring[2] == 9.0).all()) and not bool(ring[4].any()))


@pytest.mark.parametrize("taps", [2, 4, 8])
def test_short_entries_side_by_side_in_a_step_of_many(taps):
    """Entries of one to nine tokens back to back (they begin and end anywhere in the blocks' pieces), large steps (longer
    pieces), each from its own ring."""
    from sharpinference_amd import ops

    W = 24
    g = torch.Generator().manual_seed(taps)
    rng = random.Random(taps)
    for total in (60, 300, 1500):
        lens = []
        while sum(lens) < total:
            lens.append(rng.choice([1, 1, 2, 3, 4, 5, 7, 9, 40]))
        n = len(lens)
        starts = [rng.choice([0, 1, 2, taps - 1, 50]) for _ in lens]
        seqs = [torch.randn(s + m, W, generator=g) for s, m in zip(starts, lens)]
        cw = torch.randn(W, taps, generator=g)
        ring = torch.zeros(n, taps, W)
        for i, (s, x) in enumerate(zip(starts, seqs)):
            for p in range(max(0, s - taps + 1), s):
                ring[i, p % taps] = x[p]
        ring = ring.to(DEV)
        ctx = _Step(lens, starts, list(range(n)))
        h = torch.cat([x[s:] for s, x in zip(starts, seqs)]).to(DEV)
        got = ops.residual_conv(h, cw.to(DEV), ring, ctx, torch.float32).cpu()
        want = torch.cat([(x.double() + P.causal_conv(x.double(), cw.double()))[s:] for s, x in zip(starts, seqs)])
        assert _rel_rms(got, want) < FLOAT_KERNEL
        for i, x in enumerate(seqs):
            for p in range(max(0, len(x) - taps + 1), len(x)):
                assert torch.equal(ring[i, p % taps].cpu(), x[p]), (total, i)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mul_prev, mul_cur, buckets", [(29, 11, 53), (1000003, 999983, 97), (0, 1, 5), (1, 0, 200), (3, 2, 1)])
def test_the_embedding_of_token_pairs_remembers_the_previous_token(dtype, mul_prev, mul_cur, buckets):
    from sharpinference_amd import ops

    V, W = 50000, 24
    g = torch.Generator().manual_seed(buckets)
    table, pairs = torch.randn(V, W, generator=g).to(DT[dtype]), torch.randn(buckets + 1, W, generator=g).to(DT[dtype])
    ids = {r: torch.randint(0, V, (n, 1), generator=g) for r, n in TOTAL.items()}
    before = torch.full((5, 2), 123, dtype=torch.int32, device=DEV)

    def call(x, ctx):
        ctx.token_ids = x[:, 0].to(torch.int32)
        return ops.embed_bigram(ctx, table.to(DEV), pairs.to(DEV), mul_prev, mul_cur, before, 1.5)

    got = _over_plan(ids, call)
    for r in TOTAL:
        toks = ids[r][:, 0].tolist()
        want = table[toks].double() * 1.5 + pairs[P.bigram_rows(toks, mul_prev, mul_cur, buckets)].double()
        assert _rel_rms(got[r], want) < 1e-6, r
    assert before[2].tolist() == [123, 123] and before[4].tolist() == [123, 123]


# ---------------------------------------------------------------------------
# latent attention: query latents, YaRN's magnitude, sliding windows
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dn, dr, R, Rq, rot", [(3, 24, 8, 40, 20, (500.0, 8, 4.0, 64, 8.0, 1.0)), (4, 16, 16, 32, 72, (1e4, 6, 2.0, 32, 4.0, 1.0)),
                                                   (2, 8, 32, 64, 300, (1e6, 32, 40.0, 1024, 32.0, 1.0))])
def test_latent_rows_query_latents_and_rotated_parts_with_yarns_magnitude(dtype, H, dn, dr, R, Rq, rot):
    from sharpinference_amd import ops
    from sharpinference_amd.parts.position import YarnRotary, YarnScaling

    T, ps, pages, eps = 11, 16, 5, 1e-5
    g = torch.Generator().manual_seed(H)
    D = R + dr
    src = torch.randn(T, Rq + 5 + D, generator=g).to(DT[dtype])
    pos = torch.tensor([0, 1, 2, 15, 16, 17, 100, 1000, 31, 32, 5], dtype=torch.int32)
    slots = torch.tensor([3, 17, 40, -1, 79, 0, 5, 6, 7, 8, 9], dtype=torch.int32)
    nw, qw = 0.5 + torch.rand(R, generator=g), 0.5 + torch.rand(Rq, generator=g)
    scaling = dict(zip(("factor", "original", "fast", "slow"), rot[2:]))
    y = YarnRotary(dr, rot[0], YarnScaling(**scaling), "interleaved", rot[1])
    freq = y.table(torch.device(DEV))
    rows = torch.zeros(pages, 1, ps, D, dtype=DT[dtype], device=DEV)
    common = (pos.to(DEV), freq, nw.to(DEV), eps, H, dn, dr, R)
    cq = ops.latent_prep(None, 0, Rq + 5, None, rows, slots.to(DEV), *common, magnitude=y.magnitude, kv=src.to(DEV),
                         q_latent=(src.to(DEV), 0, qw.to(DEV)))
    tol = FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL
    cos, sin = P.rotation(pos.long(), rot[0], rot[1], scaling, torch.float64)
    assert _rel_rms(cq, P.rms_norm(src.double()[:, :Rq], qw.double(), eps)) < tol
    flat = rows.reshape(-1, D).cpu()
    c = P.rms_norm(src.double()[:, Rq + 5:Rq + 5 + R], nw.double(), eps)
    kr = P.rotate_pairs(src.double()[:, None, Rq + 5 + R:], cos, sin)[:, 0]
    keep = slots >= 0
    assert _rel_rms(flat[slots[keep].long()][:, :R], c[keep]) < tol
    assert _rel_rms(flat[slots[keep].long()][:, R:], kr[keep]) < max(tol, 3e-4 if dtype == "float32" else tol)      # (angle at 1000: float)
    used = set(slots[keep].tolist())
    assert not flat[[i for i in range(pages * ps) if i not in used]].any()
    q = torch.randn(T, H * (dn + dr), generator=g).to(DT[dtype])
    q_full = torch.zeros(T, H * D, dtype=DT[dtype], device=DEV)
    assert ops.latent_prep(q.to(DEV), 0, None, q_full, None, None, *common, magnitude=y.magnitude) is None
    want = P.rotate_pairs(q.double().reshape(T, H, dn + dr)[..., dn:], cos, sin)
    got = q_full.cpu().reshape(T, H, D)
    assert not got[..., :R].any() and _rel_rms(got[..., R:].reshape(T, -1), want.reshape(T, -1)) < max(tol, 3e-4 if dtype == "float32" else tol)


class _Att:
    """A step of one request as the attention kernels see it: all its tokens in prompt tiles, or as listed single tokens."""

    def __init__(self, positions, tiles):
        n = len(positions)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
        self.positions, self.entry_of_token = i32(positions), i32([0] * n)
        self.n_decode, self.decode_tokens, self.n_prefill_tiles, self.prefill_tiles, self.prefill_tile_tokens = 0, None, 0, None, 64
        if tiles:
            t = [(0, o, min(64, n - o)) for o in range(0, n, 64)]
            self.prefill_tiles, self.n_prefill_tiles = i32(t), len(t)
        else:
            self.n_decode = n


class _Group:
    def __init__(self, bt, max_context):
        self.block_table, self.max_context = bt, max_context


def _window_case(H, R, dr, S, first, window, dtype, seed, marks=()):
    """S cached rows of one request (pages that no query of positions first.. sees are not held), queries at positions first ..
    S - 1.  marks: (query position, key position) pairs whose one score is made to stand out."""
    g = torch.Generator().manual_seed(seed)
    ps, D = 16, R + dr
    keys, q = torch.randn(S, D, generator=g), torch.randn(S, H, D, generator=g)
    for i, j in marks:
        keys[j] *= 3.0
        q[i] = keys[j][None] * (30.0 / keys[j].pow(2).sum()) + 0.05 * q[i]
    keys, q = keys.to(DT[dtype]), q[first:].to(DT[dtype])
    n_blocks = (S + ps - 1) // ps
    perm = torch.randperm(n_blocks + 3, generator=g)[:n_blocks]
    rows = torch.randn(n_blocks + 3, 1, ps, D, generator=g).to(DT[dtype]) * 4.0       # what other requests left in the pages
    bt = torch.full((1, n_blocks + 1), -1, dtype=torch.int32)
    gone = max(0, first - window + 1) // ps if window else 0
    for b in range(n_blocks):
        if b >= gone:
            bt[0, b] = perm[b]
            m = min(ps, S - b * ps)
            rows[perm[b], 0, :m] = keys[b * ps:b * ps + m]
    return q, keys, rows.to(DEV), bt.to(DEV)


def _plain_rows_attention(q, keys, scale, R, first, window):
    qd, kd = q.double(), keys.double()
    T, H, _ = q.shape
    mask = P.visible(keys.shape[0], window)[first:]
    out = torch.zeros(T, H, R, dtype=torch.float64)
    for h in range(H):
        s = (qd[:, h] @ kd.T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~mask, float("-inf")), -1) @ kd[:, :R]
    return out


@pytest.mark.parametrize("how", ["tiles", "singles", "float"])
@pytest.mark.parametrize("H, R, dr, S, first, window", [
    (3, 64, 16, 90, 0, 29), (8, 96, 32, 300, 0, 72), (4, 80, 16, 330, 200, 130), (16, 128, 32, 700, 650, 300), (20, 512, 64, 200, 0, 17),
    (40, 256, 32, 150, 70, 1), (5, 32, 8, 1300, 1100, 1100), (2, 48, 8, 2300, 2200, 40), (8, 96, 32, 200, 0, 5000), (1, 16, 8, 64, 0, 32)])
def test_latent_attention_behind_a_sliding_window(H, R, dr, S, first, window, how):
    """Windows below a chunk, a page and a run, beyond them, and wider than the context; contexts whose early pages are gone."""
    from sharpinference_amd import ops

    dtype = "float32" if how == "float" else "bfloat16"
    q, keys, rows, bt = _window_case(H, R, dr, S, first, window, dtype, S + H)
    scale, T = 1.3 / math.sqrt(R + dr), S - first
    ctx = _Att(list(range(first, S)), how == "tiles")
    out = ops.attention_latent(q.reshape(T, -1).to(DEV), rows, _Group(bt, S), ctx, scale, H, R, dr, window_kind=ops.WINDOW_SLIDING,
                               window=window, kernel="generic" if how == "float" else "mfma")
    want = _plain_rows_attention(q, keys, scale, R, first, window)
    assert _rel_rms(out.reshape(T, -1), want.reshape(T, -1)) < (FLOAT_KERNEL if how == "float" else BF16_KERNEL)
    if how != "float":
        gen = ops.attention_latent(q.reshape(T, -1).to(DEV), rows, _Group(bt, S), ctx, scale, H, R, dr, window_kind=ops.WINDOW_SLIDING,
                                   window=window, kernel="generic")
        assert _rel_rms(out.reshape(T, -1), gen.reshape(T, -1)) < BF16_KERNEL


@pytest.mark.parametrize("how", ["tiles", "singles", "float"])
@pytest.mark.parametrize("window", [16, 33, 72, 128, 129, 200])
def test_a_key_just_inside_the_window_counts_and_one_just_outside_does_not(window, how):
    """One score stands out for each of several queries (at page and run borders): the key window - 1 tokens back takes the
    whole softmax, the key window tokens back changes nothing."""
    from sharpinference_amd import ops

    dtype = "float32" if how == "float" else "bfloat16"
    H, R, dr, S = 4, 64, 16, 420
    at = [window + 20, 256, 257, 287, 288, 383, 384, 419]
    for back, inside in ((window - 1, True), (window, False)):
        marks = [(i, i - back) for i in at]
        q, keys, rows, bt = _window_case(H, R, dr, S, 0, window, dtype, window, marks)
        ctx = _Att(list(range(S)), how == "tiles")
        out = ops.attention_latent(q.reshape(S, -1).to(DEV), rows, _Group(bt, S), ctx, 1.0, H, R, dr, window_kind=ops.WINDOW_SLIDING,
                                   window=window, kernel="generic" if how == "float" else "mfma").cpu().reshape(S, -1)
        want = _plain_rows_attention(q, keys, 1.0, R, 0, window).reshape(S, -1)
        other = _plain_rows_attention(q, keys, 1.0, R, 0, window - 1 if inside else window + 1).reshape(S, -1)
        for i in at:
            assert _rel_rms(other[i:i + 1], want[i:i + 1]) > 0.3                     # one token's difference in the window would show
            assert _rel_rms(out[i:i + 1], want[i:i + 1]) < (FLOAT_KERNEL if how == "float" else BF16_KERNEL), i


@pytest.mark.parametrize("E, top, scale", [(6, 1, 1.5), (8, 3, 0.7), (5, 5, 2.0), (64, 6, 1.0), (2, 1, 3.0)])
@pytest.mark.parametrize("T", [1, 7, 70])
def test_router_shares_of_the_picked_scores_times_a_scale(E, top, scale, T):
    from sharpinference_amd import ops

    W = 40
    g = torch.Generator().manual_seed(E * 100 + T)
    x, wr = torch.randn(T, W, generator=g), torch.randn(E, W, generator=g) * 0.5
    ids, wts = ops.router_topk(x.to(DEV), wr.to(DEV), top, ops.GATE_SOFTMAX_PICKED, weight_scale=scale)
    want_ids, want = P.route(x.double(), wr.double(), top, scale)
    assert torch.equal(ids.cpu().long(), want_ids) and torch.allclose(wts.cpu().double(), want, atol=1e-6)


# ---------------------------------------------------------------------------
# the engine
# ---------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    from sharpinference_amd import load_config
    from sharpinference_amd.weights.loader import write_random_model

    out = {}
    for name in CONFIGS:
        d = str(tmp_path_factory.mktemp("pagonex_" + name))
        write_random_model(load_config(config(name)), d, SEEDS[name], std=0.1, std_by_suffix=STD_BY_SUFFIX)
        out[name] = d
    return out


@functools.lru_cache(maxsize=8)
def _plain_model(d):
    return P.read_config(d), P.load_weights(d, torch.float64)


def _engine(d, dtype, **kw):
    from sharpinference_amd.engine import Engine

    args = dict(dtype=dtype, device=DEV, max_num_seqs=4, kv_tokens=1024, max_model_len=1024)
    args.update(kw)
    return Engine(d, **args)


def _run(eng, reqs, steps, free=True, picks=None):
    """steps: lists of (request id, number of its next tokens).  Returns per request the logits at every position.
    ``picks`` (a dict) receives per request, for every routed layer in order, the experts and weights the
    engine's router chose at every position."""
    from sharpinference_amd.engine import StepEntry

    at = {r: 0 for r in reqs}
    logits = {r: [] for r in reqs}
    chosen = {r: [] for r in reqs}
    for step in steps:
        entries = []
        for r, n in step:
            if at[r] == 0:
                eng.add_request(r)
            entries.append(StepEntry(r, reqs[r][at[r]:at[r] + n], list(range(n))))
        trace = [] if picks is not None else None
        out = eng.step(entries, router_trace=trace).cpu()
        o = 0
        for r, n in step:
            logits[r].append(out[o:o + n])
            if trace is not None:
                chosen[r].append([(ids[o:o + n].cpu().long(), wts[o:o + n].cpu().double()) for ids, wts, _ in trace])
            o += n
            at[r] += n
            if at[r] == len(reqs[r]) and free:
                eng.free_request(r)
    if picks is not None:
        for r, parts in chosen.items():
            picks[r] = [(torch.cat([p[l][0] for p in parts]), torch.cat([p[l][1] for p in parts])) for l in range(len(parts[0]))]
    return {r: torch.cat(v) for r, v in logits.items()}


@functools.lru_cache(maxsize=64)
def _plain_logits(d, toks):
    cfg, w = _plain_model(d)
    return P.forward(cfg, w, list(toks))


def _check(d, dtype, reqs, got, what, picks=None):
    """float32: against the plain model with its own router.  bfloat16: against the plain model run with the experts the
    engine picked (a close call between two experts falls either way once the rows are rounded)."""
    for r, toks in reqs.items():
        if dtype == "float32":
            err = _rel_rows(got[r], _plain_logits(d, tuple(toks)))
            assert float(err.max()) < FLOAT_LOGITS, f"{what}, request {r}: {float(err.max()):.2e} at row {int(err.argmax())}"
        else:
            cfg, w = _plain_model(d)
            want, noise = _noise_rows(lambda store: P.forward(cfg, w, list(toks), router_picks=picks[r] if picks else None, store=store))
            _within_noise(_rel_rows(got[r], want), noise, f"{what}, request {r}")


def _run_and_check(eng, d, dtype, reqs, steps, what):
    picks = {} if dtype == "bfloat16" else None
    got = _run(eng, reqs, steps, picks=picks)
    _check(d, dtype, reqs, got, what, picks)
    return got


def _tokens(n, vocab, seed):
    rng = random.Random(seed)
    return [rng.randrange(vocab) for _ in range(n)]


def _cuts(total, sizes):
    out, i = [], 0
    while total > 0:
        n = min(total, sizes[i % len(sizes)])
        out.append(n)
        total -= n
        i += 1
    return out


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_layers_sum_agrees_with_the_plain_model(model_dirs, name, dtype):
    """The residual sum after every layer of a 40-token prompt, in float as the engine keeps it."""
    from sharpinference_amd.engine import StepEntry

    d = model_dirs[name]
    cfg, w = _plain_model(d)
    toks = _tokens(40, CONFIGS[name]["vocab"], 9)
    eng = _engine(d, dtype)
    caught = []
    for b in eng.model.blocks:
        def fwd(stream, ctx, cache, orig=b.forward):
            orig(stream, ctx, cache)
            assert stream.h.dtype == torch.float32
            stream.settle()
            caught.append(stream.h.clone())
        b.forward = fwd
    eng.add_request("x")
    trace = []
    eng.step([StepEntry("x", toks, [39])], router_trace=trace)
    eng.free_request("x")
    picks = [(ids.cpu().long(), wts.cpu().double()) for ids, wts, _ in trace] if dtype == "bfloat16" else None

    def layers(store):
        out = []
        P.forward(cfg, w, toks, layer_outputs=out, store=store, router_picks=picks)
        return out
    want, noise = (layers(P._same), None) if dtype == "float32" else _noise_rows(layers)
    assert len(caught) == len(want)
    for i, (a, b) in enumerate(zip(caught, want)):
        if dtype == "float32":
            assert _rel_rms(a, b) < FLOAT_LOGITS, f"layer {i}: {_rel_rms(a, b):.2e}"
        else:
            _within_noise(_rel_rows(a, b), noise[i], f"layer {i}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts_portions_and_decoding_agree_with_the_plain_model(model_dirs, name, dtype):
    d = model_dirs[name]
    vocab = CONFIGS[name]["vocab"]
    eng = _engine(d, dtype)
    toks = _tokens(150, vocab, 1)
    ways = {
        "whole": [150],
        "decoded one by one": [1] * 3 + [99] + [1] * 48,          # the first tokens alone, then a tail through page borders and windows
        "portions": _cuts(150, [2, 3, 17, 2, 64, 5, 16, 1, 31]),
        "pairs": [2] * 75,
    }
    first = None
    for what, cuts in ways.items():
        got = _run_and_check(eng, d, dtype, {what: toks}, [[(what, n)] for n in cuts], f"{name} {dtype} {what}")
        if dtype == "float32":
            first = got[what] if first is None else first
            assert _rel_rms(got[what], first) < FLOAT_SAME, f"{what}: the cut changes the logits"
    assert eng.runner.graph_replays > 0                           # decode steps ran from graphs, states and all
    eng.cache.check_invariants()
    assert not eng.cache.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "even"])
def test_a_long_prompt_agrees_with_its_portions(model_dirs, name, dtype):
    """700 tokens in one step and in portions of 100: windows that have long passed, states that have moved hundreds of times."""
    d = model_dirs[name]
    toks = _tokens(700, CONFIGS[name]["vocab"], 8)
    eng = _engine(d, dtype, kv_tokens=2048)
    whole = _run_and_check(eng, d, dtype, {"w": toks}, [[("w", 700)]], f"{name} {dtype} 700 tokens at once")
    parts = _run_and_check(eng, d, dtype, {"p": toks}, [[("p", 100)] for _ in range(7)], f"{name} {dtype} 700 tokens in portions")
    if dtype == "float32":       # (in single rows a head's output nearly cancels before its norm: there the plain model run in
        same = _rel_rows(whole["w"], parts["p"])       # float32 instead of double moves by 5e-5 as well)
        assert float(same.max()) < FLOAT_LOGITS and int((same > FLOAT_SAME).sum()) <= 7


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "solo"])
def test_the_first_tokens_and_a_long_decoded_tail(model_dirs, name, dtype):
    """Every token from the first decoded alone: 260 steps (rings and states start from zeros, the windows pass over decoded
    tokens), replayed from graphs."""
    d = model_dirs[name]
    toks = _tokens(260, CONFIGS[name]["vocab"], 7)
    eng = _engine(d, dtype)
    _run_and_check(eng, d, dtype, {"x": toks}, [[("x", 1)] for _ in toks], f"decoded from the first token, {name} {dtype}")
    assert eng.runner.graph_replays >= 250
    assert all(g.pool.num_free == g.pool.num_pages for g in eng.cache.groups)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "even", "wide"])
def test_unequal_requests_in_one_batch_give_what_each_gives_alone(model_dirs, name, dtype):
    d = model_dirs[name]
    vocab = CONFIGS[name]["vocab"]
    reqs = {"a": _tokens(90, vocab, 2), "b": _tokens(37, vocab, 3), "c": _tokens(130, vocab, 4), "d": _tokens(5, vocab, 5)}
    steps = [[("a", 29), ("b", 2)], [("a", 1), ("b", 33), ("c", 64)], [("c", 2), ("a", 1), ("d", 5), ("b", 1)],
             [("a", 59), ("c", 1), ("b", 1)], [("c", 63)]]
    eng = _engine(d, dtype)
    got = _run_and_check(eng, d, dtype, reqs, steps, f"mixed {dtype}")
    if dtype == "float32":
        for r, toks in reqs.items():
            alone = _run(eng, {r: toks}, [[(r, len(toks))]])
            assert _rel_rms(got[r], alone[r]) < FLOAT_SAME, f"{r}: the batch changes the logits"
    eng.cache.check_invariants()


@pytest.mark.parametrize("name", ["odd", "even"])
def test_pages_and_slots_are_given_back_and_used_again(model_dirs, name):
    """Two state slots and a small pool serve ten requests in turn: a state, a ring or a previous token that a request before
    left in its slot, or a key in a page used again, would show."""
    d = model_dirs[name]
    vocab = CONFIGS[name]["vocab"]
    eng = _engine(d, "float32", max_num_seqs=2, kv_tokens=192, max_model_len=160, max_tokens_per_step=64)
    slots = set()
    for i in range(5):
        a, b = f"a{i}", f"b{i}"
        reqs = {a: _tokens(100 + i, vocab, 10 + i), b: _tokens(60 - i, vocab, 20 + i)}
        steps = [[(a, 40), (b, 3)], [(a, 59 + i), (b, 57 - i - 2)], [(a, 1), (b, 1)], [(b, 1)]]
        eng.add_request(a), eng.add_request(b)
        slots |= {eng.cache.requests[a].state_slot, eng.cache.requests[b].state_slot}
        eng.free_request(a), eng.free_request(b)
        got = _run(eng, reqs, steps)
        _check(d, "float32", reqs, got, f"round {i}")
        eng.cache.check_invariants()
    for g in eng.cache.groups:
        assert g.pool.total_allocs > 2 * g.pool.num_pages and g.pool.num_free == g.pool.num_pages
    assert len(slots) == 2


def test_shared_rows_serve_a_reader_with_a_wider_window_than_their_owners(model_dirs):
    """'odd': layer 0 looks back 29 tokens, layer 2 reads the same rows and looks back 41.  Decoding past both with a pool that
    gives pages back as soon as it may: the logits stay the plain model's, and a model whose reader had layer 0's window
    would differ."""
    d = model_dirs["odd"]
    cfg, w = _plain_model(d)
    toks = _tokens(130, CONFIGS["odd"]["vocab"], 12)
    eng = _engine(d, "float32", max_num_seqs=1, kv_tokens=144, max_model_len=144, max_tokens_per_step=16)
    got = _run(eng, {"x": toks}, [[("x", 16)]] * 4 + [[("x", 1)]] * 66)["x"]
    assert _rel_rms(got, P.forward(cfg, w, toks)) < FLOAT_LOGITS
    narrow = json.loads(json.dumps(cfg))
    narrow["layers"][2]["mixer"]["mask"]["size"] = 29
    assert _rel_rms(got[60:], P.forward(narrow, w, toks)[60:]) > 5e-3


def test_what_the_design_adds_would_show_if_left_out(model_dirs):
    """The weights of these tests make each mechanism matter: the plain model without it is far from the engine,
    the plain model with it is not."""
    d = model_dirs["odd"]
    cfg, w = _plain_model(d)
    toks = _tokens(80, CONFIGS["odd"]["vocab"], 6)
    eng = _engine(d, "float32")
    got = _run(eng, {"x": toks}, [[("x", 50)], [("x", 30)]])["x"]
    assert _rel_rms(got, P.forward(cfg, w, toks)) < FLOAT_LOGITS

    def changed(what):
        c = json.loads(json.dumps(cfg))
        ww = dict(w)

        def each(suffix, f):
            hit = [k for k in w if k.endswith(suffix)]
            assert hit, suffix
            for k in hit:
                ww[k] = f(w[k])

        latents = [l["mixer"] for l in c["layers"] if l["type"] == "latent_attention"]
        moes = [l["mlp"] for l in c["layers"] if l["mlp"]]

        def ident(t):
            o = torch.zeros_like(t)
            o[:, -1] = 1.0
            return o
        if what == "no bigram":
            each("bigram", torch.zeros_like)
        elif what == "the first token's bigram row like any other":
            ww["bigram"] = w["bigram"].clone()
            ww["bigram"][-1] = 0.0
        elif what == "no input convolutions":
            each("canon1", torch.zeros_like), each("canon2", torch.zeros_like)
        elif what == "input convolutions of the current token alone":
            each("canon1", lambda t: ident(t) * t), each("canon2", lambda t: ident(t) * t)
        elif what == "no norm biases":
            each("norm1.b", torch.zeros_like), each("norm2.b", torch.zeros_like), each("final.norm.b", torch.zeros_like)
        elif what == "no short convolutions":
            each(".conv", ident)
        elif what == "one decay a head":
            each(".a2", torch.zeros_like), each(".dt_bias", lambda t: torch.full_like(t, float(t.mean())))
        elif what == "no decay":
            each(".A_log", lambda t: torch.full_like(t, -30.0))
        elif what == "every write whole":
            each("mix.b", torch.zeros_like)
        elif what == "no output gate":
            each(".g2", torch.zeros_like)
        elif what == "no window":
            for m in latents:
                m.pop("mask", None)
        elif what == "a window one token wider":
            for m in latents:
                if "mask" in m:
                    m["mask"]["size"] += 1
        elif what == "no YaRN":
            for m in latents:
                if "rot" in m:
                    m["rot"].pop("scaling")
        elif what == "another rotation base":
            for m in latents:
                if "rot" in m:
                    m["rot"]["base"] *= 5.0
        elif what == "rows of one's own":
            ww["l2.mix.uk"], ww["l2.mix.uv"] = w["l2.mix.uk"].flip(1), w["l2.mix.uv"].flip(1)
        elif what == "no query latent norm":
            each("dq.norm", torch.ones_like)
        elif what == "another expert limit":
            for f in moes:
                f["expert"]["limit"] *= 0.3
        elif what == "no shared expert":
            for f in moes:
                f.pop("shared", None)
        elif what == "no router scale":
            for f in moes:
                f["router"]["scale"] = 1.0
        elif what == "no logit scale":
            c["logit_scale"] = 1.0
        return float(_rel_rows(got, P.forward(c, ww, toks)).max())

    for what in ("no bigram", "the first token's bigram row like any other", "no input convolutions",
                 "input convolutions of the current token alone", "no norm biases", "no short convolutions", "one decay a head", "no decay",
                 "every write whole", "no output gate", "no window", "a window one token wider", "no YaRN", "another rotation base",
                 "rows of one's own", "no query latent norm", "another expert limit", "no shared expert", "no router scale", "no logit scale"):
        assert changed(what) > 5e-3, what


@pytest.mark.parametrize("name", list(CONFIGS))
def test_greedy_generation_through_the_scheduler(model_dirs, name):
    d = model_dirs[name]
    cfg, w = _plain_model(d)
    vocab = CONFIGS[name]["vocab"]
    prompts = [_tokens(n, vocab, 30 + n) for n in (5, 41, 18)]
    want = [P.generate(cfg, w, p, 8) for p in prompts]
    eng = _engine(d, "float32", max_tokens_per_step=16)          # prompts are cut into portions beside decode tokens
    got = [r.token_ids for r in eng.generate(prompts, max_new_tokens=8, temperature=0.0)]
    assert got == want
    eng.cache.check_invariants()
    assert not eng.cache.requests and eng.last_stats.steps > 8


def test_the_command_line_generates_from_this_design(model_dirs):
    d = model_dirs["odd"]
    cfg, w = _plain_model(d)
    prompt = _tokens(12, CONFIGS["odd"]["vocab"], 77)
    want = P.generate(cfg, w, prompt, 6)
    cmd = [sys.executable, os.path.join(ROOT, "bin", "sharpi-cli"), "-m", d, "--prompt-ids", " ".join(map(str, prompt)), "-n", "6",
           "--temp", "0", "--dtype", "fp32", "--repeat-penalty", "1.0", "--no-display-prompt", "--ignore-eos", "--ctx-size", "256"]
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=110)
    assert out.returncode == 0, out.stderr[-2000:]
    assert [int(t) for t in out.stdout.split() if t.lstrip("-").isdigit()][:6] == want, out.stdout


def test_the_trace_runner_replays_this_design(model_dirs, tmp_path):
    d = model_dirs["odd"]
    cfg, w = _plain_model(d)
    vocab = CONFIGS["odd"]["vocab"]
    a, b = _tokens(70, vocab, 41), _tokens(20, vocab, 42)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[33:35], "want": []}, {"id": "b", "tokens": b, "want": [19]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[35:69], "want": [33]}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[69:], "want": [0]}], "end": ["a"]}]
    out = str(tmp_path / "out")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", out,
           "--max-tokens", "128"]
    p = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    for st in steps:
        p.stdin.write(json.dumps(st) + "\n")
        p.stdin.flush()
        assert p.stdout.readline().strip() == f"done {st['step']}"
    p.stdin.close()
    assert p.wait(timeout=60) == 0
    wa, wb = P.forward(cfg, w, a), P.forward(cfg, w, b)
    read = lambda n, rows: torch.from_numpy(np.fromfile(os.path.join(out, f"{n}.f32"), dtype="<f4").reshape(rows, vocab).copy())
    assert _rel_rms(read(0, 2), wa[[0, 32]]) < FLOAT_LOGITS
    assert _rel_rms(read(1, 1), wb[[19]]) < FLOAT_LOGITS
    assert _rel_rms(read(2, 1), wa[[68]]) < FLOAT_LOGITS and _rel_rms(read(3, 1), wa[[69]]) < FLOAT_LOGITS
