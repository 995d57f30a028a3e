"""Rigodra on the GPU against the plain implementation (tests/plain_rigodra.py): every mechanism alone, then
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

import plain_rigodra as P
from tiny_rigodra import CONFIGS, SEEDS, STD_BY_SUFFIX, config

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}

# Float arithmetic against the plain model in double.  Whatever the design adds shows at 5e-3 and more when left
# out (test_what_the_design_adds_would_show_if_left_out).
FLOAT_KERNEL = 2e-5           # a row out of one kernel
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


# ---------------------------------------------------------------------------
# the norm of the sum, the embedding with a norm
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("W", [8, 68, 100, 320, 1000, 2048, 8192, 9000])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_norm_of_the_sum(W, dtype):
    """LN(alpha h + delta) over rows whose mean is far from zero, the sum back into h in float and a copy beside it."""
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(W)
    T, alpha, eps = 5, 1.7, 1e-5
    h, d = torch.randn(T, W, generator=g) + 3.0, (torch.randn(T, W, generator=g) * 2.0).to(DT[dtype])
    w, b = torch.randn(W, generator=g), torch.randn(W, generator=g)
    hd = h.to(DEV)
    out = ops.sum_norm(hd, d.to(DEV), alpha, w.to(DEV), b.to(DEV), eps, DT[dtype])
    want = P.layer_norm(alpha * h.double() + d.double(), w.double(), b.double(), eps)
    assert _rel_rms(hd, want) < FLOAT_KERNEL and torch.equal(out, hd.to(DT[dtype])) and out.dtype == DT[dtype]
    h2 = h.to(DEV)
    assert ops.sum_norm(h2, d.to(DEV), alpha, w.to(DEV), b.to(DEV), eps) is None and torch.equal(h2, hd)


@pytest.mark.parametrize("W", [68, 128, 2048])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("k", [1, 3, 6])
def test_a_sum_of_experts_with_identity_picks(W, dtype, k):
    """Picks beyond the experts add the token's own row: from h in float inside the norm, from a tensor in the norm and in the
    kernel that forms the sum.  Rows of y that belong to identity picks hold NaN: nobody may read them."""
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(W + k)
    T, E, I, alpha, eps = 9, 4, 3, 0.6, 1e-5
    ids = torch.stack([torch.randperm(E + I, generator=g)[:k] for _ in range(T)])
    ids[0], ids[1] = torch.arange(k) % E if k <= E else ids[0], ids[1]
    ids[2, 0] = E + I - 1
    wts = torch.rand(T, k, generator=g)
    y = torch.randn(T * k, W, generator=g).to(DT[dtype])
    y[(ids >= E).reshape(-1)] = float("nan")
    pos = torch.arange(T * k, dtype=torch.int32)
    shared = torch.randn(T, W, generator=g).to(DT[dtype])
    h = torch.randn(T, W, generator=g)
    x = h.to(DT[dtype])
    w, b = torch.randn(W, generator=g), torch.randn(W, generator=g)
    own = (ids >= E)[:, :, None]

    def plain(ident):
        rows = torch.where(own, ident.double()[:, None], torch.nan_to_num(y.double()).reshape(T, k, W))
        return (wts.double()[:, :, None] * rows).sum(1) + shared.double()
    dev = lambda t: t.to(DEV)
    es = ops.ExpertSum(dev(y), dev(pos), dev(shared), T, k, dev(wts), (dev(ids.to(torch.int32)), E, dev(x)))
    tol = FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL
    assert _rel_rms(es.tensor(), plain(x)) < tol
    for same in (True, False):
        hd = dev(h)
        ops.sum_norm(hd, es, alpha, dev(w), dev(b), eps, DT[dtype], identity_is_h=same)
        want = P.layer_norm(alpha * h.double() + plain(h if same else x), w.double(), b.double(), eps)
        assert _rel_rms(hd, want) < FLOAT_KERNEL, same
    # the kernels that form plain sums on the fly form this one first
    one = ops.add_rmsnorm(dev(h), es, None, eps, torch.float32)
    u = h.double() + plain(x)
    assert _rel_rms(one, u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)) < tol


@pytest.mark.parametrize("W", [68, 256, 3000])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_embedding_with_a_norm(W, dtype):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(W)
    table = (torch.randn(31, W, generator=g) + 0.5).to(DT[dtype])
    w, b = torch.randn(W, generator=g), torch.randn(W, generator=g)
    ids = torch.tensor([30, 0, 7, 7], dtype=torch.int32)
    h, act = ops.embed_norm(ids.to(DEV), table.to(DEV), w.to(DEV), b.to(DEV), 1e-5, 0.7, DT[dtype])
    want = P.layer_norm(table.double()[ids.long()] * 0.7, w.double(), b.double(), 1e-5)
    assert h.dtype == torch.float32 and _rel_rms(h, want) < FLOAT_KERNEL and torch.equal(act, h.to(DT[dtype]))
    h2, none = ops.embed_norm(ids.to(DEV), table.to(DEV), w.to(DEV), b.to(DEV), 1e-5, 0.7)
    assert none is None and torch.equal(h2, h)


# ---------------------------------------------------------------------------
# feed-forwards without a gate
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("n", [1, 8, 77, 4096])
def test_activations_without_a_gate(n):
    from sharpinference_amd import ops

    z = torch.linspace(-9.0, 9.0, n) if n > 1 else torch.tensor([-0.7])
    for dtype in DT:
        x = z.to(DT[dtype])
        for name, f in (("gelu", P.gelu), ("relu2", P.relu2)):
            got, want = ops.activation(x.to(DEV), name).cpu().double(), f(x.double())
            assert torch.allclose(got, want, rtol=1e-6 if dtype == "float32" else 4e-3, atol=2e-6), (name, dtype)
    # the tanh form is another function
    wide = torch.linspace(-4.0, 4.0, 999)
    assert float((ops.activation(wide.to(DEV), "gelu") - ops.activation(wide.to(DEV), "gelu_tanh")).abs().max()) > 1e-4


@pytest.mark.parametrize("act", ["relu2", "gelu"])
def test_an_activation_in_a_products_epilogue_gives_the_bits_of_the_two_kernels(act):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(3)
    dev = lambda t: t.to(torch.bfloat16).to(DEV)
    for M, N, K in ((1, 64, 128), (7, 96, 256), (30, 128, 384)):
        x, w = dev(torch.randn(M, K, generator=g)), dev(torch.randn(N, K, generator=g) * 0.2)
        for weight in (w, ops.pack_weight(w)):
            assert torch.equal(ops.linear(x, weight, torch.bfloat16, act=act), ops.activation(ops.linear(x, weight, torch.bfloat16), act))
    x, w = dev(torch.randn(200, 128, generator=g)), ops.pack_weight(dev(torch.randn(64, 128, generator=g)))
    assert torch.equal(ops.linear(x, w, torch.bfloat16, act=act), ops.activation(ops.linear(x, w, torch.bfloat16), act))
    E, I, k, W, N = 5, 2, 3, 128, 128
    stack = dev(torch.randn(E, N, W, generator=g) * 0.2)
    packed = torch.empty_like(stack)
    ops.pack_into(packed, stack)
    for T in (3, 40, 300):
        x = dev(torch.randn(T, W, generator=g))
        ids = torch.stack([torch.randperm(E + I, generator=g)[:k] for _ in range(T)]).to(torch.int32).to(DEV)
        wts = torch.rand(T, k, generator=g).to(DEV)
        rt = ops.moe_permute(ids, wts, E, identity=True)
        n = int((ids < E).sum())
        for weight in (stack, ops.PackedWeight(packed, None)):
            a = ops.grouped_linear(x, weight, rt, True, torch.bfloat16, act=act)[:n]
            assert torch.equal(a, ops.activation(ops.grouped_linear(x, weight, rt, True, torch.bfloat16)[:n].contiguous(), act))
            if T * k <= ops.PICKED_MAX_PAIRS:
                own = (ids < E).reshape(-1)
                one = ops.gemm_skinny_picked(x, weight, ids, None, False, True, False, torch.bfloat16, ungated=act)[own]
                two = ops.gemm_skinny_picked(x, weight, ids, None, False, True, False, torch.bfloat16)[own].contiguous()
                assert torch.equal(one, ops.activation(two, act))


@pytest.mark.parametrize("T", [1, 4, 20, 90, 700])
@pytest.mark.parametrize("E, I, k", [(4, 2, 3), (7, 1, 2), (1, 3, 2), (12, 4, 6)])
def test_pairs_sorted_by_expert_leave_identity_picks_out(T, E, I, k):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(T * 10 + E)
    ids = torch.stack([torch.randperm(E + I, generator=g)[:k] for _ in range(T)]).to(torch.int32)
    if T > 3:
        ids[1] = torch.arange(k, dtype=torch.int32) % I + E                # a token of identity experts alone
    wts = torch.rand(T, k, generator=g)
    rt = ops.moe_permute(ids.to(DEV), wts.to(DEV), E, identity=True)
    off, tok, w, pos = rt.offsets.cpu(), rt.sorted_token.cpu(), rt.sorted_w.cpu(), rt.inv_pos.cpu().reshape(T, k)
    assert (off[1:] - off[:-1]).tolist() == [int((ids == e).sum()) for e in range(E)]
    seen = set()
    for t in range(T):
        for j in range(k):
            e = int(ids[t, j])
            if e >= E:
                continue
            r = int(pos[t, j])
            assert off[e] <= r < off[e + 1] and int(tok[r]) == t and float(w[r]) == float(wts[t, j]) and r not in seen
            seen.add(r)
    assert len(seen) == int(off[E])
    with pytest.raises(ops.KernelError):
        ops.moe_permute(ids.to(DEV), wts.to(DEV), E, shared_group=True, identity=True)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [1, 5, 70])
@pytest.mark.parametrize("E, k, groups", [(6, 2, (3, 1)), (8, 4, (4, 2)), (10, 3, (5, 3)), (12, 3, (2, 1)), (7, 3, None), (9, 2, (9, 4)), (130, 8, (10, 4))])
def test_the_choice_by_corrected_scores_among_the_groups_with_the_largest(E, k, groups, T, dtype):
    from sharpinference_amd import ops

    W = 64
    g = torch.Generator().manual_seed(E * 100 + T)
    x, wr = torch.randn(T, W, generator=g).to(DT[dtype]), (torch.randn(E, W, generator=g) * 0.2).to(DT[dtype])
    corr = torch.randn(E, generator=g) * 0.3 - 0.5                         # (most corrected scores are negative)
    kw = dict(correction=corr.to(DEV), group_top=1)
    if groups:
        kw.update(n_groups=groups[0], keep_groups=groups[1])
    ids, wts = ops.router_topk(x.to(DEV), wr.to(DEV), k, ops.GATE_SOFTMAX, **kw)
    gd = {"count": groups[0], "keep": groups[1]} if groups else None
    want_ids, want = P.route(x.double(), wr.double(), corr.double(), k, gd)
    assert torch.equal(ids.cpu().long(), want_ids) and torch.allclose(wts.cpu().double(), want, atol=1e-6)
    if groups and groups[0] < E and groups[1] < groups[0] and T == 70:     # ranking by the two largest is another choice
        two, _ = ops.router_topk(x.to(DEV), wr.to(DEV), k, ops.GATE_SOFTMAX, **{**kw, "group_top": 2})
        assert not torch.equal(two, ids)


# ---------------------------------------------------------------------------
# between projections and attention
# ---------------------------------------------------------------------------
class _Rows:
    def __init__(self, positions):
        T = len(positions)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
        self.n_entries, self.n_tokens = 1, T
        self.positions, self.entry_of_token = i32(positions), i32([0] * T)
        self.cu_tokens, self.state_slots = i32([0, T]), i32([0])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, G, d, e, r, T", [(4, 2, 16, 8, 16, 5), (6, 3, 10, 14, 4, 9), (8, 2, 64, 32, 32, 70), (2, 2, 128, 64, 2, 3), (1, 1, 22, 5, 8, 130)])
def test_norms_half_rotation_and_mixed_values_on_their_way_into_the_cache(H, G, d, e, r, T, dtype):
    from sharpinference_amd import ops

    g = torch.Generator().manual_seed(H * d + T)
    qn, kn, vn = H * d, G * d, G * e
    proj = torch.randn(T, qn + kn + vn + 8, generator=g).to(DT[dtype])
    other = torch.randn(T, vn + 24, generator=g).to(DT[dtype])
    wq, wk = torch.rand(d, generator=g) + 0.5, torch.rand(d, generator=g) + 0.5
    pos = [1000 + 3 * i for i in range(T)]
    slots = torch.randperm(160, generator=g)[:T].to(torch.int32)
    base, lam, eps = 700.0, 0.37, 1e-5
    freq = torch.tensor([base ** (-2.0 * i / r) for i in range(r // 2)], dtype=torch.float32)
    kc, vc = torch.zeros(10, G, 16, d, dtype=DT[dtype], device=DEV), torch.zeros(10, G, e, 16, dtype=DT[dtype], device=DEV)
    for mix in (None, (other.to(DEV), 16, lam)):
        q = ops.qk_prep(proj.to(DEV), 0, qn, qn + kn, H, G, d, e, _Rows(pos), kc, vc, slots.to(DEV), ops.NORM_PER_HEAD, wq.to(DEV), wk.to(DEV),
                        eps, freq.to(DEV), ops.PAIRS_HALF_SPLIT, v_mix=mix)
        pd = proj.double()
        cos, sin = P.rotation(torch.tensor(pos), base, r, torch.float64)
        want_q = P.rotate_halves(P.rms_norm(pd[:, :qn].reshape(T, H, d), wq.double(), eps), cos, sin)
        want_k = P.rotate_halves(P.rms_norm(pd[:, qn:qn + kn].reshape(T, G, d), wk.double(), eps), cos, sin)
        v = pd[:, qn + kn:qn + kn + vn].reshape(T, G, e)
        want_v = P.mixed_values(v, None if mix is None else other.double()[:, 16:16 + vn].reshape(T, G, e), lam)
        page, off = slots.long() // 16, slots.long() % 16
        tol = 2e-4 if dtype == "float32" else BF16_KERNEL             # (an angle at position 1,000 is known to 1,000 * 2^-24)
        assert _rel_rms(q, want_q.reshape(T, -1)) < tol
        assert _rel_rms(kc.cpu()[page, :, off].reshape(T, -1), want_k.reshape(T, -1)) < tol
        assert _rel_rms(vc.cpu()[page, :, :, off].reshape(T, -1), want_v.reshape(T, -1)) < (FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL)


# ---------------------------------------------------------------------------
# attention behind a window that keeps the first tokens, values of another width than keys, a gate a head
# ---------------------------------------------------------------------------
class _Att:
    """What the attention kernels read of a step of one request's tokens at `positions`."""

    def __init__(self, positions, tiles, tile_tokens=64):
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
        n = len(positions)
        self.positions, self.entry_of_token = i32(positions), i32([0] * n)
        self.n_decode, self.decode_tokens, self.n_prefill_tiles, self.prefill_tiles, self.prefill_tile_tokens = 0, None, 0, None, tile_tokens
        if tiles:
            t = [(0, o, min(tile_tokens, n - o)) for o in range(0, n, tile_tokens)]
            self.prefill_tiles, self.n_prefill_tiles = i32(t), len(t)
        else:
            self.n_decode = n


class _Group:
    def __init__(self, bt, max_context):
        self.block_table, self.max_context = bt, max_context


def _case(H, G, d, e, S, first, window, keep, dtype, seed, marks=(), ps=16):
    """Keys and values of one request at positions 0 .. S - 1 in pages (those that no query of positions first.. sees are gone,
    what else lies in the pool is other requests'), queries at positions first .. S - 1, gates.  marks: (query position, key
    position) pairs whose score is made to stand out, the key's values made large."""
    g = torch.Generator().manual_seed(seed)
    k, v, q = torch.randn(S, G, d, generator=g), torch.randn(S, G, e, generator=g), torch.randn(S, H, d, generator=g)
    for i, j in marks:
        k[j] *= 3.0
        v[j] *= 4.0
        for h in range(H):
            kk = k[j, h // (H // G)]
            q[i, h] = kk * (30.0 / kk.pow(2).sum()) + 0.05 * q[i, h]
    k, v, q = k.to(DT[dtype]), v.to(DT[dtype]), q[first:].to(DT[dtype])
    n_blocks = (S + ps - 1) // ps
    perm = torch.randperm(n_blocks + 3, generator=g)[:n_blocks]
    kc = (torch.randn(n_blocks + 3, G, ps, d, generator=g) * 5.0).to(DT[dtype])
    vc = (torch.randn(n_blocks + 3, G, e, ps, generator=g) * 5.0).to(DT[dtype])
    bt = torch.full((1, n_blocks + 1), -1, dtype=torch.int32)
    gone = max(0, first - window + 1) // ps if window else 0
    for b in range(n_blocks):
        if b >= gone or b < (keep + ps - 1) // ps:
            bt[0, b] = perm[b]
            m = min(ps, S - b * ps)
            kc[perm[b], :, :m] = k[b * ps:b * ps + m].transpose(0, 1)
            vc[perm[b], :, :, :m] = v[b * ps:b * ps + m].permute(1, 2, 0)
    gates = torch.randn(S - first, H + 5, generator=g).to(DT[dtype])
    return q, k, v, kc.to(DEV), vc.to(DEV), bt.to(DEV), gates


def _plain_attention(q, k, v, scale, first, mask, gates=None):
    T, H, _ = q.shape
    G = k.shape[1]
    ok = P.visible(k.shape[0], mask)[first:]
    out = torch.zeros(T, H, v.shape[2], dtype=torch.float64)
    for h in range(H):
        s = (q[:, h].double() @ k[:, h // (H // G)].double().T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~ok, float("-inf")), -1) @ v[:, h // (H // G)].double()
        if gates is not None:
            out[:, h] *= torch.sigmoid(gates[:, 2 + h].double())[:, None]
    return out.reshape(T, -1)


def _attend(how, q, kc, vc, bt, S, first, window, keep, scale, H, G, d, e, gates=None, tile_tokens=64):
    from sharpinference_amd import ops

    T = S - first
    qd, kind = q.reshape(T, -1).to(DEV), ops.WINDOW_SLIDING if window else ops.WINDOW_NONE
    gate = None if gates is None else (gates.to(DEV), 2)
    ctx = _Att(list(range(first, S)), how == "tiles", tile_tokens)
    if how == "float":
        return ops.attention_generic(qd, kc, vc, bt, ctx.entry_of_token, ctx.positions, kind, window or 0, scale, H, G, d, e, keep=keep, gate=gate)
    assert ops.decode_attention_ok(q.dtype, d, e) and ops.prefill_attention_ok(q.dtype, d, e)
    return ops.attention(qd, kc, vc, _Group(bt, S), ctx, kind, window or 0, scale, H, G, d, e, keep=keep, gate=gate)


HOW = [("float32", "float"), ("bfloat16", "float"), ("bfloat16", "tiles"), ("bfloat16", "singles")]


@pytest.mark.parametrize("dtype, how", HOW)
@pytest.mark.parametrize("H, G, d, e, S, first, window, keep", [
    (8, 2, 128, 64, 300, 0, 72, 4), (4, 2, 64, 32, 200, 0, 48, 17), (2, 1, 96, 48, 330, 100, 33, 1), (3, 3, 32, 128, 150, 0, 40, 40),
    (16, 1, 64, 128, 700, 640, 300, 32), (20, 1, 192, 128, 90, 0, 1, 2), (2, 2, 128, 128, 520, 0, 256, 33), (4, 4, 32, 32, 1700, 1600, 1000, 300),
    (6, 2, 160, 96, 260, 200, 17, 100), (4, 1, 128, 192, 100, 0, 5000, 3), (8, 4, 96, 128, 130, 0, None, 0), (5, 5, 64, 64, 2100, 2070, 20, 16)])
def test_attention_behind_a_window_that_keeps_the_first_tokens(H, G, d, e, S, first, window, keep, dtype, how):
    """Kept tokens that end inside a block, at a block's and a page's edge, beyond the window; windows of one token, below a
    chunk and beyond the context; contexts whose pages between the two are gone."""
    q, k, v, kc, vc, bt, gates = _case(H, G, d, e, S, first, window, keep, dtype, S + H)
    scale = 1.4 / math.sqrt(d)
    mask = {"size": window, "keep_first": keep} if window else None
    for gg in (gates, None):
        want = _plain_attention(q, k, v, scale, first, mask, gg)
        out = _attend(how, q, kc, vc, bt, S, first, window, keep, scale, H, G, d, e, gg)
        assert _rel_rms(out, want) < (FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL)
    if how == "tiles":                                   # a row's bits do not depend on the tile it came in
        half = _attend(how, q, kc, vc, bt, S, first, window, keep, scale, H, G, d, e, None, tile_tokens=128)
        assert _rel_rms(half, want) < BF16_KERNEL and torch.equal(half, out)


@pytest.mark.parametrize("dtype, how", HOW)
@pytest.mark.parametrize("ps", [16, 64])
@pytest.mark.parametrize("window, keep", [(16, 1), (33, 4), (48, 16), (72, 5), (64, 32), (129, 40)])
def test_keys_at_the_edges_of_window_and_kept_tokens(window, keep, ps, dtype, how):
    """One score stands out for each of several queries, at page, chunk and run borders: the key window - 1 tokens back and the
    last kept one take the whole softmax, the key window tokens back and the first that is not kept change nothing."""
    H, G, d, e, S = 4, 2, 64, 32, 460
    at = [window + keep + 40, 256, 257, 287, 288, 303, 304, 459]
    for what, key, inside in (("window", lambda i: i - window + 1, True), ("window", lambda i: i - window, False),
                              ("kept", lambda i: keep - 1, True), ("kept", lambda i: keep, False)):
        marks = [(i, key(i)) for i in at] if what == "window" else [(i, key(i)) for i in at[:1]]
        rows = [i for i, _ in marks]
        q, k, v, kc, vc, bt, _ = _case(H, G, d, e, S, 0, window, keep, dtype, window + keep, marks, ps)
        if what == "kept":                               # the other queries look for the same key
            for i in at[1:]:
                q[i] = q[at[0]]
            rows = at
        out = _attend(how, q, kc, vc, bt, S, 0, window, keep, 1.0, H, G, d, e)
        want = _plain_attention(q, k, v, 1.0, 0, {"size": window, "keep_first": keep})
        step = -1 if inside else 1
        other = _plain_attention(q, k, v, 1.0, 0, {"size": window + (step if what == "window" else 0), "keep_first": keep + (step if what == "kept" else 0)})
        for i in rows:
            assert _rel_rms(other[i:i + 1], want[i:i + 1]) > 0.3, (what, inside, i)                # one token's difference would show
            assert _rel_rms(out[i:i + 1], want[i:i + 1]) < (FLOAT_KERNEL if dtype == "float32" else BF16_KERNEL), (what, inside, i)


@pytest.mark.parametrize("how", ["tiles", "singles"])
def test_long_contexts_walk_their_pages_past_the_table_a_wave_holds(how):
    """4,000 tokens behind a window of 3,000 that keeps 70: more pages than a wave's registers hold, a jump from the kept
    tokens' pages to the window's, more than one run of the decode kernel."""
    H, G, d, e, S, first, window, keep = 2, 1, 32, 64, 4000, 3900, 3000, 70
    q, k, v, kc, vc, bt, gates = _case(H, G, d, e, S, first, window, keep, "bfloat16", 5, marks=[(3999, 69), (3950, 951), (3960, 2000)])
    want = _plain_attention(q, k, v, 1.0 / math.sqrt(d), first, {"size": window, "keep_first": keep}, gates)
    out = _attend(how, q, kc, vc, bt, S, first, window, keep, 1.0 / math.sqrt(d), H, G, d, e, gates)
    assert _rel_rms(out, want) < BF16_KERNEL


def test_the_value_widths_the_matrix_core_kernels_take():
    from sharpinference_amd import ops

    bf = torch.bfloat16
    for d, e in ((128, 64), (64, 128), (192, 128), (96, 48), (128, 128)):
        assert ops.decode_attention_ok(bf, d, e) and ops.prefill_attention_ok(bf, d, e)
    assert not ops.decode_attention_ok(bf, 10, 14) and not ops.prefill_attention_ok(bf, 128, 80) and not ops.decode_attention_ok(torch.float32, 128, 64)


# ---------------------------------------------------------------------------
# the engine
# ---------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    from sharpinference_amd import load_config
    from sharpinference_amd.weights.loader import write_random_model

    out = {}
    for name in CONFIGS:
        d = str(tmp_path_factory.mktemp("rigodra_" + name))
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
    assert eng.runner.graph_replays > 0                           # decode steps ran from graphs
    eng.cache.check_invariants()
    assert not eng.cache.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "even"])
def test_a_long_prompt_agrees_with_its_portions(model_dirs, name, dtype):
    """700 tokens in one step and in portions of 100: windows that have long passed, kept tokens far behind."""
    d = model_dirs[name]
    toks = _tokens(700, CONFIGS[name]["vocab"], 8)
    eng = _engine(d, dtype, kv_tokens=2048)
    whole = _run_and_check(eng, d, dtype, {"w": toks}, [[("w", 700)]], f"{name} {dtype} 700 tokens at once")
    parts = _run_and_check(eng, d, dtype, {"p": toks}, [[("p", 100)] for _ in range(7)], f"{name} {dtype} 700 tokens in portions")
    if dtype == "float32":
        assert _rel_rms(whole["w"], parts["p"]) < FLOAT_SAME


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "solo"])
def test_the_first_tokens_and_a_long_decoded_tail(model_dirs, name, dtype):
    """Every token from the first decoded alone: 260 steps (the kept tokens are decoded ones, the windows pass over decoded
    tokens), replayed from graphs."""
    d = model_dirs[name]
    toks = _tokens(260, CONFIGS[name]["vocab"], 7)
    eng = _engine(d, dtype)
    _run_and_check(eng, d, dtype, {"x": toks}, [[("x", 1)] for _ in toks], f"decoded from the first token, {name} {dtype}")
    assert eng.runner.graph_replays >= 250
    assert all(g.pool.num_free == g.pool.num_pages for g in eng.cache.groups)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "even", "latents"])
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
    """Two slots and a small pool serve ten requests in turn: a key or a value that a request before left in a page used
    again would show."""
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


def test_decoding_with_a_small_pool_gives_back_pages_between_the_kept_and_the_window(model_dirs):
    """'odd' with pools as small as one request needs: every page behind a window goes back except the kept tokens', which later
    queries still read; a second request then takes the same pages."""
    d = model_dirs["odd"]
    cfg, w = _plain_model(d)
    eng = _engine(d, "float32", max_num_seqs=1, kv_tokens=208, max_model_len=200, max_tokens_per_step=16)
    for seed in (12, 13):
        toks = _tokens(190, CONFIGS["odd"]["vocab"], seed)
        got = _run(eng, {"x": toks}, [[("x", 16)]] * 4 + [[("x", 1)]] * 126, free=False)["x"]
        assert _rel_rms(got, P.forward(cfg, w, toks)) < FLOAT_LOGITS
        held = {g.key: sum(p >= 0 for p in eng.cache.block_table("x", i)) for i, g in enumerate(eng.cache.groups)}
        assert held[("kv", 2, 29, 3)] <= 1 + 3 and held[("kv", 2, 40, 21)] <= 2 + 4 and held[("kv", 2, 31)] <= 3
        eng.free_request("x")
    eng.cache.check_invariants()


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

        attn = [l["mixer"] for l in c["layers"] if l["type"] == "attention"]
        latents = [l["mixer"] for l in c["layers"] if l["type"] == "latent_attention"]
        moes = [l["mlp"] for l in c["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"]
        if what == "no alpha":
            c["postln_alpha"] = 1.0
        elif what == "no embedding norm weight":
            each("embed.norm", torch.ones_like)
        elif what == "no norm biases":
            each("norm1.b", torch.zeros_like), each("norm2.b", torch.zeros_like), each("final.norm.b", torch.zeros_like)
        elif what == "no query and key norm weights":
            each("mix.q.norm", torch.ones_like), each("mix.k.norm", torch.ones_like)
        elif what == "no gate":
            each("mix.g", torch.zeros_like)
        elif what == "no kept tokens":
            for m in attn:
                m.get("mask", {}).pop("keep_first", None)
        elif what == "one kept token fewer":
            for m in attn:
                if m.get("mask", {}).get("keep_first"):
                    m["mask"]["keep_first"] -= 1
        elif what == "one kept token more":
            for m in attn:
                if m.get("mask", {}).get("keep_first"):
                    m["mask"]["keep_first"] += 1
        elif what == "no window":
            for m in attn + latents:
                m.pop("mask", None)
        elif what == "a window one token wider":
            for m in attn:
                if "mask" in m:
                    m["mask"]["size"] += 1
        elif what == "a latent window one token wider":
            latents[0]["mask"]["size"] += 1
        elif what == "no rotation":
            for m in attn:
                m.pop("rot", None)
        elif what == "no latent rotation":
            for m in latents:
                m.pop("rot", None)
        elif what == "no value mixing":
            each(".vmix", torch.zeros_like)
        elif what == "the first layer's values for all":
            each(".vmix", torch.ones_like)
        elif what == "no query latent norm":
            each("dq.norm", lambda t: t.flip(0))
        elif what == "no correction":
            each(".correction", torch.zeros_like)
        elif what == "no groups":
            for f in moes:
                f["router"].pop("groups", None)
        elif what == "experts in the identity experts' place":
            for f in moes:
                if f["router"].get("identity"):
                    n = f["router"].pop("identity")
                    f["router"]["experts"] += n
            for i, l in enumerate(cfg["layers"]):
                if l["mlp"] and l["mlp"]["kind"] == "moe":
                    r = l["mlp"]["router"]
                    for j in range(r.get("identity", 0)):
                        for part in ("up", "down"):
                            ww[f"l{i}.mlp.e{r['experts'] + j}.{part}"] = w[f"l{i}.mlp.e0.{part}"]
        elif what == "no shared expert":
            for f in moes:
                f.pop("shared", None)
        return float(_rel_rows(got, P.forward(c, ww, toks)).max())

    small = {}
    for what in ("no alpha", "no embedding norm weight", "no norm biases", "no query and key norm weights", "no gate", "no kept tokens",
                 "one kept token fewer", "one kept token more", "no window", "a window one token wider", "a latent window one token wider",
                 "no rotation", "no latent rotation", "no value mixing", "the first layer's values for all", "no query latent norm", "no correction",
                 "no groups", "experts in the identity experts' place", "no shared expert"):
        if changed(what) <= 5e-3:
            small[what] = changed(what)
    assert not small, small


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
