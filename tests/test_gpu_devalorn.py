"""The Devalorn mechanisms of the layer-list host layer (include/mi355_hybrid.h) against the float64 oracle of oracle/devalorn.py: every
new mechanism alone through its C entry point (the step between two layers with both norms and the mixtures of neighbouring tokens, products
whose segments read different operands, the low-rank decay, the recurrence with a bonus as a scan and by pieces, norms per head behind it,
the query temperature, attention with a linear distance bias or a gate per head and kept first tokens, with keys that stand out on both sides
of every edge), then whole models through the step engine -- whole prompts against token-by-token decoding, portions down to two tokens,
unequal batches against each request alone, pages and slots that are freed and used again, long decoding, the first tokens, sizes that are
1 or equal, absent parts -- greedy generation through run_engine and the scheduler, and the trace runner on a checkpoint folder.
Configurations and weights are made here."""
import json
import math
import os
import struct
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")

from oracle import devalorn as D                        # noqa: E402

pytestmark = pytest.mark.gpu
F32, BF16 = 0, 2


def _gpu():
    if not torch.cuda.is_available():
        pytest.fail("GPU tests need a visible MI355X")


def _st():
    return torch.cuda.current_stream().cuda_stream


def dev(a, dt=np.float32):
    return torch.from_numpy(np.ascontiguousarray(np.asarray(a).astype(dt))).cuda()


def bits(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def dev_dt(a, dtype):
    return dev(a) if dtype == F32 else torch.from_numpy(bits(a).view(np.int16)).cuda()


def host_dt(t, dtype):
    if dtype == F32:
        return t.cpu().numpy().astype(np.float64)
    u = t.cpu().numpy().view(np.uint16).astype(np.uint32) << 16
    return u.view(np.float32).astype(np.float64)


def empty_dt(shape, dtype):
    return torch.zeros(shape, dtype=torch.float32 if dtype == F32 else torch.int16, device="cuda")


_KEEP = []


def P(a, dt=np.float32):
    t = dev(a, dt)
    _KEEP.append(t)
    return t.data_ptr()


def PD(a, dtype):
    t = dev_dt(a, dtype)
    _KEEP.append(t)
    return t.data_ptr()


def ok(rc):
    assert rc == 0, rc
    torch.cuda.synchronize()
    _KEEP.clear()


def f32(a):
    return np.asarray(a, np.float32).astype(np.float64)


def tol(dtype, f=2e-5, b=1.5e-2):
    return f if dtype == F32 else b


def _scatter(n_rows, bs, rng):
    """a block table that uses the pool's pages in a random order, and the slot of every token row"""
    nb = -(-n_rows // bs)
    table = rng.permutation(nb + 3)[:nb].astype(np.int32)
    slots = np.array([table[t // bs] * bs + t % bs for t in range(n_rows)], np.int64)
    return table, slots, nb + 3


# ------------------------------------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("W,mixes,top", [(64, 5, 0), (37, 5, 2), (2048, 5, 3), (300, 2, 0), (40, 0, 2), (1, 5, 1), (128, 0, 0), (1030, 1, 4), (9000, 5, 0)])
def test_step_between_two_layers_over_portions(lib, dtype, W, mixes, top):
    """x' = x + both outputs (dense, the weighted rows of experts, or one of them), both norms and every mixture of a token with the one
    before it, in one launch: two unequal sequences in portions of 1, 2, 70 ... tokens, the h before a portion from the slot, zeros at a
    sequence's start whatever its slot held; then only the sum (behind the last layer) and only the norms (in front of the first)"""
    _gpu()
    rng = np.random.default_rng(W + mixes)
    lens, slots_of = [79, 9], [2, 0]
    cuts = [(1, 3), (2, 1), (70, 0), (1, 4), (5, 1)]
    n1, n2 = f32(1 + 0.2 * rng.standard_normal(W)), f32(1 + 0.2 * rng.standard_normal(W))
    mu = f32(rng.uniform(0, 1, (max(mixes, 1), W)))
    X, Y1, Y2 = ([f32(s * rng.standard_normal((n, W))) for n in lens] for s in (3, 1, 1))
    rows, pos, wt = f32(rng.standard_normal((50, W))), [rng.integers(0, 50, (n, max(top, 1))) for n in lens], [f32(rng.uniform(-1, 1, (n, max(top, 1)))) for n in lens]
    new = [X[i] + Y1[i] + ((wt[i][:, :, None] * rows[pos[i]]).sum(1) if top else Y2[i]) for i in range(2)]
    h = [D.unit_rms(x, 1e-5) * n1 for x in new]
    want_mix = [D.token_mixes(a, mu) for a in h]
    stride = W + 3
    state = dev(7 * rng.standard_normal((3, stride)))
    big = 30.0 if W == 1 else 1.0
    at = [0, 0]
    for step in cuts:
        part = [(i, at[i], c) for i, c in enumerate(step) if c]
        cat = lambda a: np.concatenate([a[i][lo:lo + c] for i, lo, c in part])      # noqa: E731
        T, cu = sum(c for _, _, c in part), np.cumsum([0] + [c for _, _, c in part])
        seg = T * W + 8
        out1, out2, o2f = empty_dt((max(1, mixes + 1) * seg,), dtype), empty_dt((T, W), dtype), torch.zeros((T, W), device="cuda")
        xo, last = torch.zeros((T, W), device="cuda"), torch.zeros((len(part), W), device="cuda")
        sl, tok_seq = np.array([slots_of[i] for i, _, _ in part]), np.concatenate([[n] * c for n, (_, _, c) in enumerate(part)])
        ok(lib.mi355_hyb_pair_step(P(cat(X)), P(cat(Y1)), None if top else P(cat(Y2)), P(rows) if top else None, P(cat(pos), np.int32), P(cat(wt)), top,
                                   xo.data_ptr(), P(n1), P(n2), out1.data_ptr(), seg, out2.data_ptr(), dtype, o2f.data_ptr(), P(mu) if mixes else None, mixes,
                                   state.data_ptr(), stride, last.data_ptr(), P([lo + c for _, lo, c in part], np.int32), P(cu, np.int32), P(sl, np.int32),
                                   P(tok_seq, np.int32), T, W, 1e-5, _st()))
        got = host_dt(out1, dtype)
        nx = cat(new)
        assert np.abs(xo.cpu().numpy() - nx).max() < 2e-6 * max(1.0, np.abs(nx).max())
        h2 = D.unit_rms(nx, 1e-5) * n2
        assert np.abs(o2f.cpu().numpy() - h2).max() < 2e-5 * big * max(1.0, np.abs(h2).max())
        assert np.abs(host_dt(out2, dtype) - h2).max() < tol(dtype, 2e-5, 1e-2) * big * max(1.0, np.abs(h2).max())
        for m in range(mixes + 1):
            w = cat(h) if m == 0 else cat([x[m - 1] for x in want_mix])
            assert np.abs(got[m * seg:m * seg + T * W].reshape(T, W) - w).max() < tol(dtype, 3e-5, 1e-2) * big * max(1.0, np.abs(w).max()), m
        if mixes:
            tail = np.stack([h[i][lo + c - 1] for i, lo, c in part])
            assert np.abs(last.cpu().numpy() - tail).max() < 2e-5 * big * max(1.0, np.abs(tail).max())
            for n, s in enumerate(sl):                                    # (in a model the recurrence's launch moves the rows)
                state[s, :W] = last[n]
        for i, _, c in part:
            at[i] += c
    assert at == lens
    x = dev(X[0])
    ok(lib.mi355_hyb_pair_step(x.data_ptr(), P(Y1[0]), None, None, None, None, 0, x.data_ptr(), None, None, None, 0, None, F32, None, None, 0, None, 0, None, None,
                               None, None, None, lens[0], W, 1e-5, _st()))
    assert np.abs(x.cpu().numpy() - (X[0] + Y1[0])).max() < 2e-6 * np.abs(X[0]).max()
    out1 = empty_dt((lens[0], W), dtype)
    ok(lib.mi355_hyb_pair_step(P(X[0]), None, None, None, None, None, 0, None, P(n1), None, out1.data_ptr(), 0, None, dtype, None, None, 0, None, 0, None, None,
                               None, None, None, lens[0], W, 1e-5, _st()))
    want = D.unit_rms(X[0], 1e-5) * n1
    assert np.abs(host_dt(out1, dtype) - want).max() < tol(dtype, 2e-5, 1e-2) * big * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,k,segs,first", [(3, 40, (128, 128, 256), 0), (1, 2080, (256, 128), 1), (20, 72, (128, 128), 0), (50, 33, (128, 384), 1), (130, 64, (256, 128, 128), 0),
                                            (70, 40, (128,) * 8, 0)])
def test_products_whose_segments_read_different_operands(lib, dtype, T, k, segs, first):
    """every product kernel (stream, tile, LDS tile, f32): segment i of the columns multiplies operand first + i"""
    _gpu()
    rng = np.random.default_rng(k)
    n, stride = sum(segs), T * (k + 8)
    a, w, b = rng.standard_normal((first + len(segs), T, k + 8)), rng.standard_normal((n, k)) / math.sqrt(k), f32(rng.standard_normal(n))
    a, w = (f32(a), f32(w)) if dtype == F32 else (D.bf16_round(a), D.bf16_round(w))
    ends = np.cumsum((0,) + segs)
    want = np.concatenate([a[first + i][:, :k] @ w[ends[i]:ends[i + 1]].T for i in range(len(segs))], axis=1) + b
    out = torch.zeros((T, n), device="cuda")
    rows = np.array(segs, np.int32)
    ok(lib.mi355_hyb_linear_segments(out.data_ptr(), n, PD(a, dtype), dtype, k + 8, stride, first, PD(w, dtype), P(b), rows.ctypes.data, len(segs), T, n, k, dtype, _st()))
    assert np.abs(out.cpu().numpy() - want).max() < 2e-5 * max(1.0, np.abs(want).max())
    bad = np.array([n - 100, 100], np.int32)                              # a segment that ends inside a tile; segments that do not add up
    assert lib.mi355_hyb_linear_segments(out.data_ptr(), n, P(b), F32, k, 0, 0, P(b), None, bad.ctypes.data, 2, T, n, k, F32, _st()) != 0
    assert lib.mi355_hyb_linear_segments(out.data_ptr(), n, P(b), F32, k, 0, 0, P(b), None, rows.ctypes.data, len(segs), T, n + 128, k, F32, _st()) != 0
    _KEEP.clear()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,ff,k", [(3, 16, 24), (1, 48, 2080), (12, 160, 2048), (20, 80, 40), (50, 112, 33), (130, 144, 64), (200, 64, 96), (65, 16, 32)])
def test_gate_and_up_in_one_product(lib, dtype, T, ff, k):
    """interleaved gate and up rows, every product kernel: act(gate) up with silu and gelu, results in f32 or bf16"""
    _gpu()
    rng = np.random.default_rng(ff)
    rnd = f32 if dtype == F32 else D.bf16_round
    a, w = rnd(rng.standard_normal((T, k + 8))), rnd(rng.standard_normal((2 * ff, k)) * 1.5 / math.sqrt(k))
    il = empty_dt((2 * ff, k), dtype)
    ok(lib.mi355_hyb_interleave_gate_up(il.data_ptr(), PD(w, dtype), 1, ff, k, dtype, _st()))
    order = [h * ff + b * 16 + j for b in range(ff // 16) for h in (0, 1) for j in range(16)]
    assert np.array_equal(host_dt(il, dtype), w[order])
    z = a[:, :k] @ w.T
    gelu = lambda x: 0.5 * x * (1 + np.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x ** 3)))     # noqa: E731
    for act, fn in ((1, D.silu), (2, gelu)):
        for out_dt in ((F32,) if dtype == F32 else (F32, BF16)):
            out = empty_dt((T, ff + 3), out_dt)
            ok(lib.mi355_hyb_linear_glu(out.data_ptr(), out_dt, ff + 3, PD(a, dtype), k + 8, il.data_ptr(), T, ff, k, act, dtype, _st()))
            want, got = fn(z[:, :ff]) * z[:, ff:], host_dt(out, out_dt)
            assert np.abs(got[:, :ff] - want).max() < tol(out_dt, 3e-5, 8e-3) * max(1.0, np.abs(want).max()) and (got[:, ff:] == 0).all(), (act, out_dt)
    assert lib.mi355_hyb_linear_glu(il.data_ptr(), dtype, ff, il.data_ptr(), k, il.data_ptr(), T, ff + 8, k, 1, dtype, _st()) != 0
    assert lib.mi355_hyb_linear_glu(il.data_ptr(), dtype, ff, il.data_ptr(), k, il.data_ptr(), T, ff, k, 3, dtype, _st()) != 0


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W,E,top,ff", [(5, 64, 6, 2, 32), (70, 64, 4, 3, 96), (300, 96, 3, 2, 64), (1, 32, 9, 9, 16), (40, 40, 7, 2, 24)])
def test_grouped_gate_up_experts(lib, dtype, T, W, E, top, ff):
    """grouping, gate and up with silu behind them in one product (ff a multiple of 16; else two launches), the down product and the
    weighted sum of the rows equal every expert run alone"""
    _gpu()
    rng = np.random.default_rng(T + E)
    h, gu, dn = D.bf16_round(rng.standard_normal((T, W))), D.bf16_round(rng.standard_normal((E, 2 * ff, W)) / math.sqrt(W)), D.bf16_round(rng.standard_normal((E, W, ff)) / math.sqrt(ff))
    ids = np.stack([rng.permutation(E)[:top] for _ in range(T)])
    wt = f32(rng.uniform(0.1, 1, (T, top)))
    want = np.zeros((T, W))
    for t in range(T):
        for e, w in zip(ids[t], wt[t]):
            a = D.silu(gu[e, :ff] @ h[t]) * (gu[e, ff:] @ h[t])
            want[t] += w * (dn[e] @ (a if dtype == F32 else D.bf16_round(a)))
    pairs = T * top
    bm = min(lib.mi355_hyb_moe_block_rows(pairs, E, 2 * ff, W, dtype), lib.mi355_hyb_moe_block_rows(pairs, E, W, ff, dtype))
    nb = (pairs + bm - 1) // bm + E
    pos, tokrow, table = (torch.zeros(n, dtype=torch.int32, device="cuda") for n in (pairs, nb * bm, 2 * nb))
    ok(lib.mi355_hyb_moe_group(pos.data_ptr(), tokrow.data_ptr(), table.data_ptr(), P(ids, np.int32), pairs, top, E, bm, nb, _st()))
    act, y, hd, gud = empty_dt((nb * bm, ff), dtype), torch.zeros((nb * bm, W), device="cuda"), dev_dt(h, dtype), dev_dt(gu, dtype)
    if ff % 16 == 0:
        il = torch.zeros_like(gud)
        ok(lib.mi355_hyb_interleave_gate_up(il.data_ptr(), gud.data_ptr(), E, ff, W, dtype, _st()))
        ok(lib.mi355_hyb_linear_grouped_glu(act.data_ptr(), dtype, ff, hd.data_ptr(), W, tokrow.data_ptr(), il.data_ptr(), 2 * ff * W, table.data_ptr(), bm, nb, ff, W, 1,
                                            dtype, _st()))
    else:
        z = torch.zeros((nb * bm, 2 * ff), device="cuda")
        ok(lib.mi355_hyb_linear_grouped(z.data_ptr(), 2 * ff, hd.data_ptr(), dtype, W, tokrow.data_ptr(), gud.data_ptr(), 2 * ff * W, table.data_ptr(), bm, nb, 2 * ff, W, dtype,
                                        _st()))
        ok(lib.mi355_hyb_silu_glu(act.data_ptr(), dtype, z.data_ptr(), nb * bm, ff, table.data_ptr(), bm, _st()))
    ok(lib.mi355_hyb_linear_grouped(y.data_ptr(), W, act.data_ptr(), dtype, ff, None, PD(dn, dtype), W * ff, table.data_ptr(), bm, nb, W, ff, dtype, _st()))
    got = (wt[:, :, None] * y.cpu().numpy()[pos.cpu().numpy().reshape(T, top)]).sum(1)
    assert np.abs(got - want).max() < tol(dtype, 2e-5, 2e-2) * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("T,rank,C", [(1, 1, 7), (3, 6, 96), (5, 64, 300), (70, 70, 256), (200, 130, 33), (65, 5, 513)])
def test_low_rank_decay(lib, T, rank, C):
    _gpu()
    rng = np.random.default_rng(rank)
    z, w2, w0 = f32(2 * rng.standard_normal((T, rank + 3))), f32(rng.standard_normal((C, rank)) / math.sqrt(rank)), f32(rng.uniform(-7, 2, C))
    out = torch.full((T, C + 2), -5.0, device="cuda")
    ok(lib.mi355_hyb_lowrank_decay(out.data_ptr(), C + 2, P(z), rank + 3, P(w2.T), P(w0), T, rank, C, _st()))
    got = out.cpu().numpy()
    want = -np.exp(np.tanh(z[:, :rank]) @ w2.T + w0)
    assert (np.abs(got[:, :C] - want) < 1e-5 * np.abs(want)).all() and (got[:, C:] == -5.0).all()
    x = f32(rng.standard_normal((T, 12)))                                 # the oracle's map from the mixture on: w1 first
    w1 = f32(rng.standard_normal((rank, 12)))
    ok(lib.mi355_hyb_lowrank_decay(out.data_ptr(), C + 2, P(x @ w1.T), rank, P(w2.T), P(w0), T, rank, C, _st()))
    assert np.abs(np.exp(out.cpu().numpy()[:, :C].astype(np.float64)) - D.lowrank_decay(x, w1, w2, w0)).max() < 2e-5


@pytest.mark.parametrize("heads,d,vd,pieces", [(4, 24, 16, 0), (3, 5, 1, 0), (2, 64, 24, 0), (1, 200, 80, 0), (2, 400, 20, 0), (2, 64, 64, 0), (4, 32, 16, 1), (2, 16, 48, 1),
                                               (3, 128, 128, 1), (1, 256, 144, 1), (2, 48, 32, 1), (1, 512, 16, 1), (2, 64, 64, 1), (2, 80, 80, 1)])
def test_bonus_recurrence_over_portions_and_reused_slots(lib, heads, d, vd, pieces):
    """two unequal sequences side by side in portions (of 1, 2, 63, 64, 65, 190 ... tokens) that continue from their slots, as a scan and
    by pieces on the matrix cores; decays per token and channel from none at all to the whole state at once, mixed within a piece; stale
    slots (position 0 starts from zero), a slot used again; the row that travels with the state"""
    _gpu()
    rng = np.random.default_rng(heads * 1000 + d)
    ld, row_n, n_slots = heads * (2 * d + vd) + 4, 37, 3
    stride = heads * d * vd + row_n + 8
    r_off, k_off, v_off = 4, 4 + heads * d, 4 + 2 * heads * d
    u = f32(rng.standard_normal((heads, d)))
    state = dev(rng.standard_normal((n_slots, stride)))
    row_ptr = state.data_ptr() + 4 * (heads * d * vd)

    def make(T):
        x = f32(rng.standard_normal((T, ld)) / math.sqrt(math.sqrt(d)))
        lw = -np.exp(rng.uniform(-7, 1, (T, heads * d)) - 5.0 * (rng.random((1, heads * d)) < 0.4))
        lw[rng.random(lw.shape) < 0.02] = -1e4                            # the channel forgets everything
        lw[:, rng.random(heads * d) < 0.1] = 0.0                          # the channel forgets nothing
        lw[:, 0] = np.where(np.arange(T) % 7 == 0, -90.0, -1e-4)          # and both in turn
        lw = f32(lw)
        o, Sf = D.bonus_recurrence(x[:, r_off:k_off].reshape(T, heads, d), x[:, k_off:v_off].reshape(T, heads, d), x[:, v_off:].reshape(T, heads, vd),
                                   np.exp(lw).reshape(T, heads, d), u)
        return x, lw, o, Sf

    def run(seqs, rows):
        """seqs: [(projection rows, log decays, slot, context length behind the portion)]"""
        cu = np.cumsum([0] + [len(s[0]) for s in seqs])
        T = int(cu[-1])
        o = torch.zeros((T, heads, vd), device="cuda")
        n = lib.mi355_hyb_bonus_recurrence_scratch(max(T, 640), 1, heads, d, vd) if pieces else 0
        scratch = torch.full((max(n, 1),), float("nan"), device="cuda")
        ok(lib.mi355_hyb_bonus_recurrence(o.data_ptr(), state.data_ptr(), stride, P(np.concatenate([s[0] for s in seqs])), ld, r_off, k_off, v_off,
                                          P(np.concatenate([s[1] for s in seqs])), heads * d, P(u), P([s[3] for s in seqs], np.int32), P(cu, np.int32),
                                          P([s[2] for s in seqs], np.int32), len(seqs), T, heads, d, vd, P(rows), row_ptr, row_n,
                                          scratch.data_ptr() if pieces else None, _st()))
        for s, r in zip(seqs, rows):
            assert np.array_equal(state[s[2], heads * d * vd:heads * d * vd + row_n].cpu().numpy(), r.astype(np.float32))
        return o.cpu().numpy()
    cutsA, cutsB = ([1, 2, 63, 64, 65, 190, 1], [3, 1, 1, 130, 0, 2, 64]) if pieces else ([1, 2, 9, 1, 27], [3, 1, 1, 12, 0])
    A, B = make(sum(cutsA)), make(sum(cutsB))
    la = lb = 0
    gotA, gotB = [], []
    for ca, cb in zip(cutsA, cutsB):
        seqs = [(A[0][la:la + ca], A[1][la:la + ca], 2, la + ca)] + ([(B[0][lb:lb + cb], B[1][lb:lb + cb], 0, lb + cb)] if cb else [])
        o = run(seqs, f32(rng.standard_normal((len(seqs), row_n))))
        gotA.append(o[:ca]); gotB.append(o[ca:])
        la += ca; lb += cb
    for got, ref in ((np.concatenate(gotA), A), (np.concatenate(gotB), B)):
        assert np.abs(got - ref[2]).max() < 3e-5 * max(1.0, np.abs(ref[2]).max())
    st = state.cpu().numpy()
    for slot, ref in ((2, A), (0, B)):
        assert np.abs(st[slot, :heads * d * vd].reshape(heads, d, vd) - ref[3]).max() < 3e-5 * max(1.0, np.abs(ref[3]).max())
    C = make(70 if pieces else 6)                                          # a new sequence in A's slot: nothing of A is left
    assert np.abs(run([(C[0], C[1], 2, len(C[0]))], f32(rng.standard_normal((1, row_n)))) - C[2]).max() < 3e-5 * max(1.0, np.abs(C[2]).max())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,heads,vd", [(4, 3, 20), (70, 2, 64), (1, 1, 1), (3, 5, 130)])
def test_norm_per_head_with_weights_of_its_own_and_gate(lib, dtype, T, heads, vd):
    _gpu()
    rng = np.random.default_rng(vd)
    n = heads * vd
    o, z, w = f32(3 * rng.standard_normal((T, heads, vd))), f32(rng.standard_normal((T, n + 5))), f32(1 + 0.3 * rng.standard_normal(n))
    out = empty_dt((T, n + 6), dtype)
    ok(lib.mi355_hyb_gated_norm_heads(out.data_ptr(), dtype, n + 6, 4, P(o), P(w), vd, P(z), n + 5, 0, T, heads, vd, 1e-5, 0.7, _st()))
    want = D.head_norm_gate(o, w, D.silu(z[:, :n]), 1e-5) * 0.7
    got = host_dt(out, dtype)
    assert np.abs(got[:, 4:4 + n] - want).max() < tol(dtype, 2e-5, 8e-3) * max(1.0, np.abs(want).max()) and (got[:, :4] == 0).all() and (got[:, 4 + n:] == 0).all()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,H,G,d,vd,coef,every,cached", [(5, 4, 2, 16, 16, 0.5, 3, 1), (3, 3, 1, 20, 7, 0.0, 1, 1), (90, 6, 3, 32, 48, 1.25, 16, 1), (4, 2, 2, 8, 8, 0.7, 1, 0),
                                                          (2, 16, 4, 128, 128, 0.1, 100, 1), (7, 1, 1, 1, 1, 2.0, 5, 0)])
def test_whole_projection_norm_and_query_temperature(lib, dtype, T, H, G, d, vd, coef, every, cached):
    """one norm over all of q (and of k), the temperature of positions on both sides of its steps, keys and values in their pages -- or
    nothing cached at all (a layer that reads another layer's pages)"""
    _gpu()
    rng = np.random.default_rng(d + T)
    nq, nk, nv = H * d, G * d, G * vd
    src = f32(2 * rng.standard_normal((T, nq + nk + nv + 3)))
    qw, kw = f32(1 + 0.3 * rng.standard_normal(nq)), f32(1 + 0.3 * rng.standard_normal(nk))
    pos = np.arange(T) + (every - 2 if every > 2 else 0)
    pos[-1] = 40 * every - 1
    slots = rng.permutation(T + 5)[:T]
    qo, kp, vp = empty_dt((T, nq), dtype), empty_dt((T + 5, nk), dtype), empty_dt((T + 5, nv), dtype)
    ok(lib.mi355_hyb_attn_prepare_whole_temp(qo.data_ptr(), kp.data_ptr() if cached else None, vp.data_ptr() if cached else None, P(src), nq + nk + nv + 3, 0, nq, nq + nk,
                                             P(qw), P(kw), P(pos, np.int64), P(slots, np.int64), T, H, G, d, vd, 0, coef, float(every), 1e-5, dtype, _st()))
    temp = D.query_temperature(int(pos.max()) + 1, coef, every)[pos]
    want = D.unit_rms(src[:, :nq], 1e-5) * qw * temp[:, None]
    big = 20.0 if d == 1 else 1.0
    assert np.abs(host_dt(qo, dtype) - want).max() < tol(dtype, 2e-5, 8e-3) * big * np.abs(want).max()
    k, v = host_dt(kp, dtype), host_dt(vp, dtype)
    if cached:
        wk = D.unit_rms(src[:, nq:nq + nk], 1e-5) * kw
        assert np.abs(k[slots] - wk).max() < tol(dtype, 2e-5, 8e-3) * big * np.abs(wk).max()
        assert np.abs(v[slots] - src[:, nq + nk:nq + nk + nv]).max() < tol(dtype, 1e-6, 8e-3) * np.abs(src).max()
    else:
        assert (k == 0).all() and (v == 0).all()
    # the form with a rotation and norms per head takes the temperature too
    half = d // 2
    rot = 2 * half
    if rot and T < 50:
        ang = np.arange(int(pos.max()) + 1)[:, None] * 50.0 ** (-2.0 * np.arange(half) / rot)
        qo2 = empty_dt((T, nq), dtype)
        ok(lib.mi355_hyb_attn_prepare_temp(qo2.data_ptr(), None, None, P(src), nq + nk + nv + 3, 0, 0, 0, None, None, P(np.cos(ang)), P(np.sin(ang)), P(pos, np.int64),
                                           P(slots, np.int64), T, H, G, d, vd, rot, 0, 0, None, coef, float(every), 1e-5, dtype, _st()))
        full = np.zeros((int(pos.max()) + 1, H, d))
        full[pos] = src[:, :nq].reshape(T, H, d)
        want = D.rotate_halves(full, 50.0, rot)[pos] * temp[:, None, None]
        assert np.abs(host_dt(qo2, dtype).reshape(T, H, d) - want).max() < tol(dtype, 2e-5, 8e-3) * np.abs(want).max()


def _edges(L, first, bs, window, keep):
    """(query, key) pairs: the window's first key, the last one before it, the last kept token, the first not kept, page borders, itself"""
    out = []
    for i in sorted({L - 1, first, first + 1, first + (L - first) // 2} & set(range(first, L))):
        w = window or L
        out += [(i, j) for j in (i - w + 1, i - w, i - w + 2, keep - 1, keep, 0, 1, i, i // bs * bs, i // bs * bs - 1) if 0 <= j <= i]
    return sorted(set(out))


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("H,G,d,vd,bs,L,n_new,window,keep,biased", [
    (4, 2, 16, 16, 16, 300, 1, 128, 0, 1), (4, 2, 16, 24, 16, 257, 1, 43, 7, 0), (6, 3, 12, 5, 8, 290, 7, 50, 0, 1), (3, 3, 20, 20, 8, 90, 40, 1, 0, 1), (3, 3, 20, 20, 8, 90, 40, 1, 3, 0),
    (3, 3, 32, 32, 64, 330, 130, 100, 0, 1), (8, 2, 64, 64, 32, 400, 400, 97, 33, 0), (6, 2, 32, 48, 16, 270, 80, 16, 0, 1), (4, 4, 128, 64, 64, 640, 1, 512, 0, 1),
    (4, 1, 128, 128, 64, 520, 64, 200, 70, 0), (2, 2, 64, 128, 16, 150, 150, 70, 0, 1), (6, 3, 96, 192, 16, 200, 100, 30, 9, 0), (4, 2, 32, 160, 16, 200, 100, 64, 17, 0), (4, 1, 128, 256, 16, 230, 150, 64, 17, 0),
    (4, 2, 64, 256, 32, 200, 140, 90, 0, 1), (4, 1, 64, 64, 64, 260, 200, 0, 0, 1), (1, 1, 1, 1, 16, 70, 5, 20, 2, 0), (5, 1, 16, 16, 16, 130, 66, 1000, 0, 1)])
def test_attention_with_keys_that_stand_out(lib, dtype, H, G, d, vd, bs, L, n_new, window, keep, biased):
    """the last n_new tokens of a sequence of L against its scattered pages (the generic kernel, the matrix-core kernels with one wave per
    head and with grouped heads, values up to twice as wide as the keys): a linear distance bias, or kept first tokens and a gate per
    head; ONE (query, key) pair at a time whose score stands out, so that every edge shows alone"""
    _gpu()
    rng = np.random.default_rng(H * 100 + d + n_new + window)
    first, scale = L - n_new, 0.8 / math.sqrt(d)
    table, slots, nblk = _scatter(L, bs, rng)
    slopes = D.distance_slopes(H) if biased else None
    gate = None if biased else f32(2 * rng.standard_normal((n_new, H + 3)))
    q0, k0, v = rng.standard_normal((L, H, d)), rng.standard_normal((L, G, d)), rng.standard_normal((L, G, vd))
    rnd = f32 if dtype == F32 else D.bf16_round
    v = rnd(v)
    mask = D.window_mask(L, window, keep)
    pairs = _edges(L, first, bs, window, keep)
    if len(pairs) > 12:
        pairs = [pairs[i] for i in sorted(rng.choice(len(pairs), 12, replace=False))]
    shown = 0
    for pair in [None] + pairs:
        q, k = q0.copy(), k0.copy()
        if pair:                                                          # the pair's score stands 25 above the bias it pays
            i, j = pair
            u = rng.standard_normal(d); u /= np.linalg.norm(u)
            k[j] = 4.0 * u
            for h in range(H):
                q[i, h] = u * (25.0 + (slopes[h] * (i - j) if biased else 0.0)) / (4.0 * scale)
        q, k = rnd(q), rnd(k)
        want = D.grouped_attention(q, k, v, scale, mask, f32(slopes) if biased else None)[first:]
        if pair and mask[pair] and d > 1:
            shown += np.abs(want[pair[0] - first, 0] - v[pair[1], 0]).max() < 0.2
        want = want * 0.9 * (D.sigmoid(gate[:, :H])[:, :, None] if gate is not None else 1.0)
        kp, vp = np.zeros((nblk * bs, G * d)), np.zeros((nblk * bs, G * vd))
        kp[slots], vp[slots] = k.reshape(L, -1), v.reshape(L, -1)
        out, tok_seq = torch.zeros((n_new, H * vd + 2), device="cuda"), torch.zeros(n_new, dtype=torch.int32, device="cuda")
        ok(lib.mi355_hyb_attention_ex(out.data_ptr(), F32, H * vd + 2, 2, PD(q[first:], dtype), PD(kp, dtype), PD(vp, dtype), P(table, np.int32), P([L], np.int32),
                                      P([0, n_new], np.int32), tok_seq.data_ptr(), None, P(np.concatenate([slopes, np.zeros(H)])) if biased else None, 1,
                                      P(gate) if gate is not None else None, H + 3, 1, n_new, H, G, d, vd, bs, len(table), 0, window, keep, scale, 0.9, 0, 0, 0.0, 0, dtype,
                                      _st()))
        got = out.cpu().numpy()[:, 2:].reshape(n_new, H, vd)
        assert np.abs(got - want).max() < tol(dtype, 1e-4, 3e-2) * max(1.0, np.abs(want).max()), pair
    assert shown >= 2 or d == 1


# ------------------------------------------------------------------------------------------------------------ whole models
def _moe(E, top, ff, scale=1.0):
    return {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": E, "scale": scale, "top": top}}


def _dense(ff):
    return {"ff": ff, "kind": "dense"}


def _par(heads, kv, dim, vdim, window, keep, rot, rheads, rdim, ls=1.2, rs=0.8, scale=None):
    left = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": scale or 1.3 * dim ** -0.5, "vdim": vdim}
    if window:
        left["mask"] = {"keep_first": keep, "size": window}
    if rot:
        left["rot"] = {"base": 3000.0, "dims": rot}
    return {"left": left, "left_scale": ls, "right": {"dim": rdim, "heads": rheads}, "right_scale": rs}


def _att(heads, kv, dim, vdim, window, temp=(0.5, 16), kv_from=None, scale=None):
    c = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": scale or 1.3 * dim ** -0.5, "vdim": vdim}
    if window:
        c["mask"] = {"size": window}
    if temp:
        c["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if kv_from is not None:
        c["kv_from"] = kv_from
    return c


def _layer(mixer, mlp):
    return {"type": "parallel" if "left" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def small_config(variant):
    if variant == 0:        # both mixers and feed-forwards, sizes that are not each other's equals, two layers on one layer's keys and values
        layers = [_layer(_att(4, 2, 16, 24, 21), _dense(72)), _layer(_par(6, 2, 12, 20, 9, 3, 8, 3, 16), _moe(7, 2, 24, 1.5)),
                  _layer(_att(4, 2, 16, 24, 30, (1.5, 5), 0), None), _layer(_par(2, 2, 20, 12, 33, 20, 20, 2, 20, 0.6, 1.4), _dense(40)),
                  _layer(_att(8, 2, 16, 24, 7, None, 0), _moe(5, 5, 16, 0.7))]
        return {"architecture": "Devalorn", "layers": layers, "norm": {"eps": 1e-5}, "vocab": 131, "width": 64}
    if variant == 1:        # no windows, no rotation, no kept tokens, one head pair, no feed-forward, an expert count of one, a width that is no multiple of 8
        layers = [_layer(_par(3, 3, 20, 20, 0, 0, None, 5, 8, 1.0, 1.0), None), _layer(_att(3, 1, 10, 6, 0), _moe(1, 1, 20)),
                  _layer(_par(4, 1, 8, 8, 5, 0, 4, 1, 24), _dense(33))]
        return {"architecture": "Devalorn", "layers": layers, "norm": {"eps": 1e-6}, "vocab": 90, "width": 100}
    # head sizes of the matrix-core kernels, pieces of the recurrence, windows over several pages
    layers = [_layer(_par(8, 2, 64, 64, 100, 17, 32, 4, 64), _dense(160)), _layer(_att(4, 1, 32, 32, 70, (0.5, 64)), _moe(12, 3, 64, 2.0)),
              _layer(_par(4, 2, 32, 160, 40, 5, 32, 2, 48), _moe(6, 1, 32)), _layer(_att(4, 1, 32, 32, 90, (0.2, 100), 1), _dense(96))]
    return {"architecture": "Devalorn", "layers": layers, "norm": {"eps": 1e-5}, "vocab": 257, "width": 160}


def settle_router(cfg, W, rng):
    """routing for runs in 16 bits: rounding noise flips a choice between two experts whose logits are close, and the oracle cannot follow
    such a flip.  One channel of the residual is the same large constant everywhere (the embedding puts it there, nothing writes to it),
    and the routers read it so that some experts of a layer lie far above the rest; the weights among them still come from the token.  The
    choice by token is what the f32 runs cover."""
    W["embed"][:, 0] = 4.0
    for k in W:
        if k.endswith(".o") or k.endswith(".down"):
            W[k][0] = 0.0
    for i, lc in enumerate(cfg["layers"]):
        k = "l%d.mlp.router" % i
        if k in W:
            W[k][:, 0] = 0.0
            W[k][rng.permutation(len(W[k]))[:lc["mlp"]["router"]["top"]], 0] = 16.0
            W["l%d.norm2" % i][0] = 1.0


def model_of(cfg, W, dtype, block_size=16, state_slots=4):
    from candle_vllm_amd.hybrid_model import DevalornSpec, HybridModel
    m = HybridModel(DevalornSpec(cfg, {k: v.shape for k, v in W.items()}), dtype=dtype, block_size=block_size, state_slots=state_slots)
    m.load_state_dict_f32(W)
    return m


def build(cfg, dtype, seed=0, block_size=16, state_slots=4, right_vdim=None):
    rng = np.random.default_rng(seed)
    W = D.random_devalorn(rng, cfg, right_vdim=right_vdim)
    if dtype == "bfloat16":
        settle_router(cfg, W, rng)
    return model_of(cfg, W, dtype, block_size, state_slots), W


def row_errs(a, b):
    d = a - b
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / max(1e-9, np.sqrt((b * b).mean()))


def row_err(a, b, lim=1.0):
    return (row_errs(a, b) / lim).max()


TOL = {"float32": 3e-5, "bfloat16": 4e-2}


def limits(cfg, W, toks, want, dtype):
    """the error allowed at every position.  In 16 bits the norm per head behind the recurrence multiplies the rounding of h at positions
    where a head's output is nearly zero (a first token whose r . u k is small): there, three times the largest of what five roundings of
    the sublayers' inputs (to nearest, and errors of up to half a last place at random) do to the oracle"""
    if dtype == "float32":
        return np.full(len(toks), TOL[dtype])
    rng = np.random.default_rng(0)

    def half_place(h):
        return h * (1.0 + rng.uniform(-1, 1, h.shape) / 512.0)
    noise = [row_errs(D.forward(cfg, W, toks, operand=f)[0], want) for f in [D.bf16_round] + [half_place] * 4]
    return np.maximum(TOL[dtype], 3.0 * np.max(noise, axis=0))


CLOSE_CALL = 1e-5           # a choice between two experts whose logits lie closer than this may fall either way in f32


def oracle_logits(cfg, W, toks, rng=None):
    """the oracle's logits (and trace); no routing decision of the run may be a close call -- with `rng`, tokens are drawn again"""
    for _ in range(30):
        margins = []
        out, tr = D.forward(cfg, W, toks, margins)
        if not margins or min(margins) > CLOSE_CALL:
            return out, tr, toks
        assert rng is not None, "a routing decision of this test is a close call: take other tokens"
        toks = rng.integers(0, cfg["vocab"], len(toks)).tolist()
    raise AssertionError("no token sequence without a close call")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("variant", [0, 1, 2])
def test_model_whole_portions_decode_against_oracle(lib, dtype, variant):
    """one request whole, with the residual stream behind every layer; then the same tokens in portions of 2, 1, 17, ... tokens and
    token by token: every way must give the oracle's logits at every position (the token before, the recurrent state and the
    windows cross every cut; pages of 16 tokens)"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    cfg = small_config(variant)
    m, W = build(cfg, dtype, seed=variant)
    rng = np.random.default_rng(11)
    n = 330 if variant == 2 else 75
    toks = rng.integers(0, cfg["vocab"], n).tolist()
    want, want_trace, toks = oracle_logits(cfg, W, toks, rng)
    eng = StepEngine(m, 3 * 336)
    eng.feed("a", toks)
    got, tr = eng.step(["a"], [list(range(n))], trace=True)
    eng.finish("a")
    if dtype == "float32":
        assert np.abs(tr.cpu().numpy() - want_trace).max() < 1e-4 * np.abs(want_trace).max()
    lim = limits(cfg, W, toks, want, dtype)
    assert row_err(got.cpu().numpy(), want, lim) < 1
    for cuts in ([2, 1, 17, 1, 1, 2, 30, 3, 18], [40] + [1] * 35, [1] * 20 + [55]):
        cuts = cuts + ([n - 75] if n > 75 else [])
        assert sum(cuts) == n
        lo, rows = 0, []
        for c in cuts:
            eng.feed("b", toks[lo:lo + c])
            rows.append(eng.step(["b"], [list(range(c))]).cpu().numpy())
            lo += c
        eng.finish("b")
        assert row_err(np.concatenate(rows), want, lim) < 1, cuts
        assert eng.free_pages() == eng.num_blocks and eng.be.state_free_slots() == 4


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches_pages_and_slots_reused(lib, dtype):
    """five requests of unequal length through four slots and a pool that only fits them because pages come back: portions of some
    beside single tokens of others, a request that sits steps out, a late one that takes over a freed slot and freed pages --
    every logit must equal the request run alone in the oracle"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    cfg = small_config(0)
    m, W = build(cfg, dtype, seed=3)
    rng = np.random.default_rng(21)
    lens = {"a": 70, "b": 33, "c": 5, "d": 48, "e": 41}
    toks = {r: oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], n).tolist(), rng)[2] for r, n in lens.items()}
    want = {r: D.forward(cfg, W, toks[r])[0] for r in toks}
    eng = StepEngine(m, 80 + 48 + 16 + 48 + 0)                            # "e" (48 rounded) only fits after "b" and "c" have gone
    sched = [[("a", 2), ("b", 30)], [("a", 16), ("b", 1), ("c", 3)], [("a", 1), ("b", 1), ("c", 1), ("d", 47)], [("a", 30), ("c", 1), ("b", 1)],
             [("a", 1), ("d", 1), ("e", 2)], [("e", 38), ("a", 1)], [("a", 19), ("e", 1)]]
    at, got = {r: 0 for r in toks}, {r: [] for r in toks}
    for step in sched:
        ids, w = [], []
        for r, n in step:
            eng.feed(r, toks[r][at[r]:at[r] + n])
            at[r] += n
            ids.append(r); w.append(list(range(n)))
        out = eng.step(ids, w).cpu().numpy()
        lo = 0
        for r, n in step:
            got[r].append(out[lo:lo + n]); lo += n
        for r, _ in step:
            if at[r] == lens[r]:
                eng.finish(r)
    assert at == lens
    for r in toks:
        assert row_err(np.concatenate(got[r]), want[r], limits(cfg, W, toks[r], want[r], dtype)) < 1, r
    assert eng.free_pages() == eng.num_blocks and eng.be.state_free_slots() == 4


def test_long_decoding_first_tokens_and_graph_replays(lib):
    """a prompt of one token, then 150 tokens one by one (decoding batches replay a captured hipGraph): the first tokens and every
    later one equal the oracle; the eager steps give the same logits bit for bit"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    cfg = small_config(0)
    m, W = build(cfg, "float32", seed=8)
    rng = np.random.default_rng(9)
    want, _, toks = oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], 151).tolist(), rng)
    outs = {}
    for use_graph in (True, False):
        eng = StepEngine(m, 160)
        eng.use_graph = use_graph
        rows = []
        for t in toks:
            eng.feed("a", [t])
            rows.append(eng.step(["a"]).cpu().numpy())
        eng.finish("a")
        outs[use_graph] = np.concatenate(rows)
    assert row_err(outs[True][:4], want[:4]) < TOL["float32"]
    assert row_err(outs[True], want) < TOL["float32"]
    assert np.array_equal(outs[True], outs[False])
    cap, rep = m.graph_stats()
    assert cap >= 1 and rep >= 100


def test_sizes_that_are_one(lib):
    """one head, one expert of which one is used, head sizes of one, a window of one token, one kept token, a low-rank map of rank one"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    layers = [_layer(_par(1, 1, 2, 1, 1, 1, 2, 1, 1, 1.0, 1.0), _moe(1, 1, 1)), _layer(_att(1, 1, 1, 1, 1, (1.0, 1)), _dense(1)),
              _layer(_att(1, 1, 1, 1, 3, (0.3, 2), 1), _moe(3, 3, 1)), _layer(_par(2, 1, 4, 2, 3, 1, 2, 2, 3), None)]
    cfg = {"architecture": "Devalorn", "layers": layers, "norm": {"eps": 1e-5}, "vocab": 17, "width": 32}
    rng = np.random.default_rng(5)
    W = D.random_devalorn(rng, cfg, rank=1)
    m = model_of(cfg, W, "float32")
    want, _, toks = oracle_logits(cfg, W, rng.integers(0, 17, 40).tolist(), rng)
    eng = StepEngine(m, 64)
    lo, rows = 0, []
    for c in [1, 2, 20, 1, 1, 15]:
        eng.feed("a", toks[lo:lo + c])
        rows.append(eng.step(["a"], [list(range(c))]).cpu().numpy())
        lo += c
    assert row_err(np.concatenate(rows), want) < TOL["float32"]


def sharp_model(window_left, keep, window_right, scale_up):
    """a model whose attention weights are sharp: what one key decides shows in the logits"""
    cfg = {"architecture": "Devalorn", "layers": [_layer(_par(4, 2, 32, 32, window_left, keep, 16, 2, 16, 3.0, 0.5), None),
                                                  _layer(_att(4, 2, 32, 32, window_right, (0.5, 40)), _dense(64))],
           "norm": {"eps": 1e-5}, "vocab": 200, "width": 96}
    W = D.random_devalorn(np.random.default_rng(4), cfg)
    for k in W:
        if k.endswith(".left.q") or k.endswith(".q.norm"):
            W[k] = D.bf16_round(W[k] * scale_up)
    return cfg, W


def test_windows_kept_tokens_temperature_and_gates_decide_the_logits(lib):
    """a sharp model on 64-token pages, 300 tokens, whole and decoded: right to the f32 tolerance -- and the oracle with a window one token off,
    one kept token more or less, no temperature, no distance bias, or the previous token left out of the mixtures is hundreds of
    tolerances away, so that each of them would show"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    cfg, W = sharp_model(37, 5, 70, 4.0)
    rng = np.random.default_rng(3)
    toks = rng.integers(0, cfg["vocab"], 300).tolist()
    want = D.forward(cfg, W, toks)[0]
    m = model_of(cfg, W, "float32", block_size=64)
    eng = StepEngine(m, 320)
    eng.feed("a", toks)
    assert row_err(eng.step(["a"], [list(range(300))]).cpu().numpy(), want) < TOL["float32"]
    eng.finish("a")
    eng.feed("b", toks[:230])
    got = [eng.step(["b"], [list(range(230))]).cpu().numpy()]
    for t in toks[230:]:
        eng.feed("b", [t])
        got.append(eng.step(["b"]).cpu().numpy())
    assert row_err(np.concatenate(got), want) < TOL["float32"]

    def off(change):
        c = json.loads(json.dumps(cfg))
        w = dict(W)
        change(c["layers"][0]["mixer"]["left"], c["layers"][1]["mixer"], w)
        return row_errs(D.forward(c, w, toks)[0], want).max()
    for change in (lambda l, a, w: l["mask"].update(size=36), lambda l, a, w: l["mask"].update(size=38), lambda l, a, w: l["mask"].update(keep_first=4),
                   lambda l, a, w: l["mask"].update(keep_first=6), lambda l, a, w: a["mask"].update(size=69), lambda l, a, w: a["mask"].update(size=71),
                   lambda l, a, w: a.pop("q_temp"), lambda l, a, w: w.pop("l0.mix.left.g"),
                   lambda l, a, w: w.update({k: 0 * v for k, v in w.items() if ".mu." in k})):
        assert off(change) > 100 * TOL["float32"]


def test_values_of_the_recurrence_may_be_wider_than_its_keys(lib):
    """the right branch's value size comes from its tensors"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    cfg = {"architecture": "Devalorn", "layers": [_layer(_par(2, 1, 16, 16, 30, 2, 16, 3, 16), _dense(32))], "norm": {"eps": 1e-5}, "vocab": 60, "width": 48}
    m, W = build(cfg, "float32", right_vdim=32)
    toks = np.random.default_rng(0).integers(0, 60, 100).tolist()
    want = D.forward(cfg, W, toks)[0]
    eng = StepEngine(m, 112)
    rows, lo = [], 0
    for c in (70, 1, 2, 27):
        eng.feed("a", toks[lo:lo + c])
        rows.append(eng.step(["a"], [list(range(c))]).cpu().numpy())
        lo += c
    assert row_err(np.concatenate(rows), want) < TOL["float32"]


@pytest.mark.parametrize("chunk", [0, 7])
def test_greedy_generation_through_scheduler(lib, chunk):
    """run_engine + the C++ scheduler (continuous batching, staggered arrivals, chunked prefill): every request generates exactly the
    tokens the oracle generates for it alone"""
    _gpu()
    from candle_vllm_amd import block_engine as be
    from candle_vllm_amd.engine import Request, run_engine
    cfg = small_config(0)
    m, W = build(cfg, "float32", seed=6)
    rng = np.random.default_rng(6)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (19, 3, 40, 11, 26)]
    n_new = 10
    want = []
    for p in prompts:
        seq, out = list(p), []
        for _ in range(n_new):
            lg = D.forward(cfg, W, seq)[0][-1]
            top2 = np.sort(lg)[-2:]
            assert top2[1] - top2[0] > 1e-4, "a greedy choice of this test is a close call: take another seed"
            out.append(int(lg.argmax()))
            seq.append(out[-1])
        want.append(out)
    nblk = 24
    sched = be.Scheduler(16, nblk, 0, 4, 64, prefill_chunk_size=chunk)
    sched.block_engine.state_init(4)
    m.alloc_cache(nblk)
    reqs = [Request(i, p, n_new, arrival_step=2 * i) for i, p in enumerate(prompts)]
    stats = run_engine(m, sched, reqs, chunk=chunk)
    assert stats["finished"] == len(prompts)
    for r, w in zip(reqs, want):
        assert r.tokens == w, (r.id, r.tokens, w)
    assert sched.block_engine.state_free_slots() == 4


def _write_model(folder, cfg, W):
    """config.json + model.safetensors (bf16; 8-byte header length, JSON header, data) of a configuration"""
    head, blobs, at = {}, [], 0
    for name, a in W.items():
        raw = bits(a).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    hb = json.dumps(head).encode()
    (folder / "model.safetensors").write_bytes(struct.pack("<Q", len(hb)) + hb + b"".join(blobs))
    (folder / "config.json").write_text(json.dumps(cfg))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner_replays_a_mixed_schedule_from_a_checkpoint_folder(lib, tmp_path, dtype):
    """bin/trace_run as a user starts it: a folder with config.json and model.safetensors, steps on standard input -- six requests over
    time, at most four alive, portions beside single tokens, a pool that only fits because ended requests give their pages and slots
    back -- and the logits it writes equal the oracle's for every request alone"""
    _gpu()
    cfg = small_config(2)
    rng = np.random.default_rng(17)
    W = D.random_devalorn(rng, cfg)
    if dtype == "bfloat16":
        settle_router(cfg, W, rng)
    _write_model(tmp_path, cfg, W)
    lens = {"a": 150, "b": 40, "c": 3, "d": 90, "e": 61, "f": 130}
    toks = {r: oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], n).tolist(), rng)[2] for r, n in lens.items()}
    want = {r: D.forward(cfg, W, toks[r])[0] for r in toks}
    lim = {r: limits(cfg, W, toks[r], want[r], dtype) for r in toks}
    sched = [[("a", 70), ("b", 2)], [("a", 1), ("b", 30), ("c", 3)], [("a", 64), ("b", 1), ("d", 65)], [("a", 1), ("b", 7), ("d", 1), ("e", 17)],
             [("a", 14), ("d", 24), ("e", 1), ("f", 2)], [("e", 43), ("f", 100)], [("f", 1)], [("f", 27)]]
    at, steps, rows = {r: 0 for r in toks}, [], []
    for n, step in enumerate(sched):
        entries, end, got = [], [], []
        for r, c in step:
            w = sorted(set([0, c - 1] + rng.integers(0, c, 3).tolist()))
            entries.append({"id": r, "tokens": toks[r][at[r]:at[r] + c], "want": w})
            got += [(r, at[r] + k) for k in w]
            at[r] += c
            if at[r] == lens[r]:
                end.append(r)
        steps.append(json.dumps({"step": n, "entries": entries, "end": end}))
        rows.append(got)
    assert at == lens
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "448"], input="\n".join(steps) + "\n", capture_output=True, text=True, timeout=170)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done ")] == ["done %d" % n for n in range(len(sched))]
    for n, got in enumerate(rows):
        a = np.fromfile(out / ("%d.f32" % n), "<f4").reshape(len(got), cfg["vocab"])
        ref = np.stack([want[r_][p_] for r_, p_ in got])
        assert row_err(a, ref, np.array([lim[r_][p_] for r_, p_ in got])) < 1, (n, dtype)


def random_config(rng):
    """sizes, head counts, depth, order, expert counts and constants drawn at random (sizes that are not all multiples of 16 or 32; layers
    without a feed-forward, borrowed keys and values)"""
    def mlp():
        u = rng.random()
        if u < 0.15:
            return None
        if u < 0.5:
            return _dense(int(rng.choice([24, 100, 256])))
        E = int(rng.choice([2, 5, 16, 24]))
        return _moe(E, int(rng.integers(1, min(E, 6) + 1)), int(rng.choice([16, 40, 64])), float(rng.choice([0.5, 1.0, 2.5])))
    layers = []
    for i in range(int(rng.integers(3, 7))):
        G, d = int(rng.choice([1, 2, 3])), int(rng.choice([16, 20, 32, 48, 64, 96, 128]))
        H, vd = G * int(rng.choice([1, 2, 3, 4])), int(d * rng.choice([0.5, 1, 2]))
        scale, window = float(d ** -0.5 * rng.uniform(0.7, 2.0)), int(rng.choice([5, 32, 64, 77, 130]))
        if rng.random() < 0.5:
            rot = int(rng.choice([n for n in (2, 8, 16, d) if n <= d]))
            c = _par(H, G, d, vd, window, int(rng.choice([0, 1, 4, 40])), rot, int(rng.choice([1, 2, 3, 4])), int(rng.choice([8, 16, 20, 32, 48, 64, 128])),
                     float(rng.uniform(0.5, 1.5)), float(rng.uniform(0.5, 1.5)), scale)
            c["left"]["rot"]["base"] = float(rng.choice([1e3, 1e4, 5e5]))
        else:
            temp = (float(rng.uniform(0.1, 1.0)), int(rng.choice([1, 10, 64, 200]))) if rng.random() < 0.8 else None
            own = [j for j, lc in enumerate(layers) if lc["type"] == "attention" and "kv_from" not in lc["mixer"]]
            if own and rng.random() < 0.5:
                j = int(rng.choice(own))
                b = layers[j]["mixer"]
                c = _att(b["heads"], b["kv_heads"], b["dim"], b["vdim"], window, temp, j, scale)
            else:
                c = _att(H, G, d, vd, window, temp, None, scale)
        layers.append(_layer(c, mlp()))
    return {"architecture": "Devalorn", "layers": layers, "norm": {"eps": float(rng.choice([1e-5, 1e-6]))}, "vocab": int(rng.integers(50, 600)),
            "width": int(rng.choice([64, 100, 128, 160, 256]))}


@pytest.mark.parametrize("seed", [2, 11, 21, 33, 47, 58])
def test_random_configurations_whole_and_mixed_schedules(lib, seed):
    """three unequal requests of a random configuration: each alone in one step, then together in a random schedule of portions (2, 3,
    17, 64, 65, 100 tokens; a request may sit a step out) that ends token by token -- on 64-token pages, in f32 and bf16"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    rng = np.random.default_rng(seed)
    cfg = random_config(rng)
    W = D.random_devalorn(rng, cfg)
    lens = [int(rng.integers(150, 300)), int(rng.integers(1, 40)), int(rng.integers(60, 130))]
    toks = [oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], n).tolist(), rng)[2] for n in lens]
    want = [D.forward(cfg, W, t)[0] for t in toks]
    for dtype in ("float32", "bfloat16"):
        if dtype == "bfloat16":
            settle_router(cfg, W, rng)
            want = [D.forward(cfg, W, t)[0] for t in toks]
        lim = [limits(cfg, W, t, w, dtype) for t, w in zip(toks, want)]
        m = model_of(cfg, W, dtype, block_size=64)
        eng = StepEngine(m, 64 * 10)
        for i, t in enumerate(toks):
            eng.feed("w", t)
            got = eng.step(["w"], [list(range(len(t)))]).cpu().numpy()
            eng.finish("w")
            assert row_err(got, want[i], lim[i]) < 1, (seed, dtype, "whole", i, cfg)
        at, got = [0, 0, 0], [[], [], []]
        srng = np.random.default_rng(seed + 1)
        while any(a < n for a, n in zip(at, lens)):
            ids, w, step = [], [], []
            for i in range(3):
                left = lens[i] - at[i]
                if left == 0 or srng.random() < 0.2:
                    continue
                c = 1 if left <= 8 else min(left - 8, int(srng.choice([2, 3, 17, 64, 65, 100])))
                eng.feed(str(i), toks[i][at[i]:at[i] + c])
                ids.append(str(i)); w.append(list(range(c))); step.append((i, c))
                at[i] += c
            if not ids:
                continue
            out = eng.step(ids, w).cpu().numpy()
            lo = 0
            for i, c in step:
                got[i].append(out[lo:lo + c]); lo += c
        for i in range(3):
            eng.finish(str(i))
            assert row_err(np.concatenate(got[i]), want[i], lim[i]) < 1, (seed, dtype, "mixed", i, cfg)
