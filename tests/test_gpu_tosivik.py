"""The Tosivik mechanisms of the layer-list host layer (include/mi355_hybrid.h) against the float64 oracle of oracle/tosivik.py: every
new mechanism alone through its C entry point (the step between two sublayers over several residual streams, the embedding by pairs of
tokens, products with an activation behind them, attention inside chunks over scattered pages with keys that stand out on both sides of
every edge, linear attention with a constant decay as a scan and by pieces over portions and reused slots, the biased router, the gate
behind the norm), then whole models through the step engine -- whole prompts against token-by-token decoding, portions down to two
tokens, unequal batches against each request alone, pages and slots that are freed and used again, long decoding, the first tokens,
sizes that are 1 or equal, absent parts -- greedy generation through run_engine and the scheduler, and the trace runner on a checkpoint
folder.  Configurations and weights are made here."""
import json
import math
import os
import struct
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")

from oracle import tosivik as S                         # noqa: E402

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
@pytest.mark.parametrize("streams,T,W,experts", [(1, 3, 40, 0), (2, 4, 64, 2), (3, 2, 50, 0), (4, 70, 128, 3), (5, 3, 36, 1), (8, 2, 300, 0), (11, 2, 20, 5),
                                                 (16, 3, 33, 2), (4, 2, 2048, 4), (3, 1, 1, 1)])
def test_step_between_two_sublayers(lib, dtype, streams, T, W, experts):
    """the mixing of the copies with a sublayer's output (dense, the weighted rows of experts, both), the next sublayer's input and its
    norm, in one launch: nothing computed yet, in between, and behind the last sublayer (only the sum)"""
    _gpu()
    rng = np.random.default_rng(streams * 100 + W)
    X, y = f32(3 * rng.standard_normal((T, streams, W))), f32(rng.standard_normal((T, W)))
    M, ow, iw, nw = f32(rng.standard_normal((streams, streams))), f32(rng.standard_normal(streams)), f32(rng.standard_normal(streams)), f32(1 + 0.2 * rng.standard_normal(W))
    top = max(experts, 1)
    rows, pos, wt = f32(rng.standard_normal((40, W))), rng.integers(0, 40, (T, top)), f32(rng.uniform(-1, 1, (T, top)))
    xs = X.transpose(1, 0, 2)

    def run(dense, mix, norm, want_sum):
        xd, out, out2, sm = dev(X), empty_dt((T, W), dtype), torch.zeros((T, W), device="cuda"), torch.zeros((T, W), device="cuda")
        ok(lib.mi355_hyb_stream_step(xd.data_ptr(), P(y) if dense else None, P(rows) if mix and experts else None, P(pos, np.int32), P(wt), top,
                                     P(M) if mix else None, P(ow), sm.data_ptr() if want_sum else None, P(iw) if norm else None,
                                     P(nw) if norm else None, out.data_ptr(), dtype, out2.data_ptr() if norm else None, T, streams, W, 1e-5, _st()))
        out_y = (y if dense else 0.0) + ((wt[:, :, None] * rows[pos]).sum(1) if mix and experts else 0.0) + np.zeros((T, W))
        nx = S.stream_update(xs, M, ow, out_y) if mix else xs
        big = max(1.0, np.abs(nx).max())
        if norm:
            assert np.abs(xd.cpu().numpy().transpose(1, 0, 2) - nx).max() < 2e-6 * big * streams
            h = S.rms_norm(S.stream_mixture(nx, iw), nw, 1e-5)
            assert np.abs(out2.cpu().numpy() - h).max() < 3e-5 * max(1.0, np.abs(h).max()) * (30 if W == 1 else 1)
            assert np.abs(host_dt(out, dtype) - h).max() < tol(dtype, 3e-5, 1e-2) * max(1.0, np.abs(h).max()) * (30 if W == 1 else 1)
        if want_sum:
            assert np.abs(sm.cpu().numpy() - nx.sum(0)).max() < 3e-6 * big * streams
    run(False, False, True, False)                                        # in front of the first sublayer
    run(True, True, True, False)
    run(experts == 0, True, True, True)                                   # the experts' rows alone
    run(True, True, False, True)                                          # behind the last one


def test_embedding_by_pairs_of_tokens_over_portions_and_reused_slots(lib):
    """rows of the second table for two unequal sequences side by side, in portions; the previous token crosses every cut in the state
    slot, a sequence's first token takes the last row whatever its slot held; multipliers beyond 32 bits in the product"""
    _gpu()
    rng = np.random.default_rng(4)
    V, buckets, mp, mc, stride = 50000, 65521, 1234577, 98765, 7
    state = torch.full((3, stride), 31337, dtype=torch.int32, device="cuda")

    def run(seqs):
        """seqs: [(tokens of the portion, slot, context length behind it)]"""
        toks, cu = np.concatenate([s[0] for s in seqs]), np.cumsum([0] + [len(s[0]) for s in seqs])
        rows = torch.zeros(len(toks), dtype=torch.int32, device="cuda")
        ok(lib.mi355_hyb_bigram_rows(rows.data_ptr(), state.data_ptr(), stride, P(toks, np.int32), P([s[2] for s in seqs], np.int32), P(cu, np.int32),
                                     P([s[1] for s in seqs], np.int32), len(seqs), len(toks), buckets, mp, mc, _st()))
        return rows.cpu().numpy()
    a, b = rng.integers(0, V, 600), rng.integers(0, V, 9)
    wa, wb = S.bigram_rows(a, buckets, mp, mc), S.bigram_rows(b, buckets, mp, mc)
    assert wa[0] == buckets and max(wa[1:]) < buckets
    la = lb = 0
    for ca, cb in ((1, 2), (1, 1), (2, 0), (590, 5), (6, 1)):
        seqs = [(a[la:la + ca], 2, la + ca)] + ([(b[lb:lb + cb], 0, lb + cb)] if cb else [])
        got = run(seqs)
        assert got.tolist() == wa[la:la + ca] + wb[lb:lb + cb]
        la += ca; lb += cb
    c = rng.integers(0, V, 3)
    assert run([(c, 2, 3)]).tolist() == S.bigram_rows(c, buckets, mp, mc)     # slot 2 again: nothing of `a` is left
    for dtype in (F32, BF16):
        T, W, copies, vocab = 6, 37, 3, 20
        table, big, ids, rows = S.bf16_round(rng.standard_normal((vocab, W))), S.bf16_round(rng.standard_normal((11, W))), rng.integers(0, vocab, T), rng.integers(0, 11, T)
        x = torch.zeros((T, copies, W), device="cuda")
        for bg in (True, False):
            ok(lib.mi355_hyb_embed_streams(x.data_ptr(), PD(table, dtype), PD(big, dtype) if bg else None, P(rows, np.int32),
                                           P(ids, np.int32), T, copies, W, vocab, 2.5, dtype, _st()))
            want = table[ids] * 2.5 + (big[rows] if bg else 0.0)
            assert np.abs(x.cpu().numpy() - want[:, None, :]).max() < 2e-6 * np.abs(want).max()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,n,k", [(3, 40, 24), (1, 33, 2080), (20, 70, 40), (50, 100, 33), (130, 150, 64), (200, 48, 96)])
def test_products_with_an_activation_behind_them(lib, dtype, T, n, k):
    """every product kernel (stream, tile, LDS tile, f32): the activation on all columns or the first few, results in f32 or bf16"""
    _gpu()
    rng = np.random.default_rng(n)
    a, w, b = rng.standard_normal((T, k)), rng.standard_normal((n, k)) / math.sqrt(k), f32(rng.standard_normal(n))
    a, w = (f32(a), f32(w)) if dtype == F32 else (S.bf16_round(a), S.bf16_round(w))
    z = a @ w.T + b
    ad, wd = dev_dt(a, dtype), dev_dt(w, dtype)
    for act, fn in ((0, lambda v: v), (1, S.silu), (2, S.gelu_tanh), (3, S.relu2)):
        for cols in (n, n // 3):
            for out_dt in ((F32,) if dtype == F32 else (F32, BF16)):
                out = empty_dt((T, n), out_dt)
                ok(lib.mi355_hyb_linear_act(out.data_ptr(), out_dt, n, ad.data_ptr(), dtype, k, wd.data_ptr(), P(b), T, n, k, act, cols, dtype, _st()))
                want = np.concatenate([fn(z[:, :cols]), z[:, cols:]], axis=1)
                assert np.abs(host_dt(out, out_dt) - want).max() < tol(out_dt, 2e-5, 8e-3) * max(1.0, np.abs(want).max()), (act, cols, out_dt)


def _mask_pairs(chunk, L, first, bs):
    """(query, key) pairs at the edges: the first key of the query's chunk, the last one before it, far inside, page borders, itself"""
    out = []
    for i in sorted({L - 1, first, first + 1, min(L - 1, (first // chunk + 1) * chunk), min(L - 1, (first // chunk + 1) * chunk - 1), first + (L - first) // 2} & set(range(first, L))):
        lo = i // chunk * chunk
        out += [(i, j) for j in (lo, lo - 1, lo + 1, i, i // bs * bs, i // bs * bs - 1, lo // bs * bs, 0) if 0 <= j <= i]
    return sorted(set(out))


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("Hh,G,d,rot,bs,L,n_new,chunk", [
    (4, 2, 16, 8, 16, 300, 1, 128), (4, 2, 16, 16, 16, 257, 1, 128), (4, 2, 16, 16, 16, 256, 1, 128), (4, 4, 12, 4, 16, 290, 7, 50), (3, 3, 20, 0, 8, 90, 40, 1),
    (3, 3, 32, 32, 64, 330, 130, 100), (8, 2, 64, 64, 32, 400, 400, 97), (6, 2, 32, 16, 16, 270, 80, 16), (4, 4, 128, 64, 64, 640, 1, 512), (4, 1, 128, 128, 64, 520, 64, 200),
    (2, 2, 256, 32, 16, 150, 150, 70), (5, 5, 64, 20, 64, 500, 90, 450), (3, 1, 96, 96, 32, 300, 300, 2), (4, 1, 64, 64, 64, 200, 200, 10000), (4, 1, 64, 64, 64, 260, 200, 0)])
def test_attention_inside_chunks_with_keys_that_stand_out(lib, dtype, Hh, G, d, rot, bs, L, n_new, chunk):
    """the last n_new tokens of a sequence of L against its scattered pages (the generic kernel, the matrix-core kernels with one wave per
    head and with grouped heads): queries get ONE key whose score stands out -- first of their chunk, last of the chunk before (which
    must not be seen), page borders, the first token -- one pair at a time, so that every edge shows alone.  Keys and queries turn,
    the cached values are the keys as projected"""
    _gpu()
    rng = np.random.default_rng(Hh * 100 + d + n_new + chunk)
    first, scale, T0 = L - n_new, 0.8 / math.sqrt(d), L
    r = {"base": 300.0, "dims": rot, "scaling": {"factor": 5.0, "fast": 8.0, "original": 64, "slow": 1.0}}
    ang, amp = S.yarn_angles(r, T0) if rot else (np.zeros((T0, 0)), 1.0)
    table, slots, nblk = _scatter(L, bs, rng)
    nq, nk = Hh * d, G * d
    q0, k0 = rng.standard_normal((L, Hh, d)), rng.standard_normal((L, G, d))
    pairs = [None] + _mask_pairs(chunk or 10 ** 6, L, first, bs)
    if len(pairs) > 12:
        pairs = [None] + [pairs[1 + i] for i in sorted(rng.choice(len(pairs) - 1, 11, replace=False))]
    for pair in pairs:
        q, k = q0.copy(), k0.copy()
        if pair:                                                          # score of the pair = 25, far above the rest: aligned behind the rotation
            i, j = pair
            u = rng.standard_normal(d); u /= np.linalg.norm(u)
            for x, t, heads in ((q, i, Hh), (k, j, G)):
                v = math.sqrt(25.0 / scale) * np.tile(u, (1, heads, 1))
                x[t] = S.rotate_halves(v, -ang[t:t + 1], 1.0 / amp, rot)[0] if rot else v[0]
        q, k = (f32(q), f32(k)) if dtype == F32 else (S.bf16_round(q), S.bf16_round(k))
        qr, kr = (S.rotate_halves(q, ang, amp, rot), S.rotate_halves(k, ang, amp, rot)) if rot else (q, k)
        if dtype == BF16:
            qr, kr = S.bf16_round(qr), S.bf16_round(kr)
        want = S.softmax_attention(qr, kr, k, scale, S.chunk_mask(L, chunk))[first:]
        src = np.concatenate([q.reshape(L, nq), k.reshape(L, nk)], axis=1)
        qo, kp, vp = empty_dt((L, nq), dtype), empty_dt((nblk * bs, nk), dtype), empty_dt((nblk * bs, nk), dtype)
        ok(lib.mi355_hyb_attn_prepare_ex(qo.data_ptr(), kp.data_ptr(), vp.data_ptr(), P(src), nq + nk, 0, nq, nq, None, None, P(np.cos(ang) * amp) if rot else None,
                                         P(np.sin(ang) * amp) if rot else None, P(np.arange(L), np.int64), P(slots, np.int64), L, Hh, G, d, d, rot, 0, 0, None, 1e-5,
                                         dtype, _st()))
        qn, out, tok_seq = qo[first:].contiguous(), torch.zeros((n_new, Hh * d), device="cuda"), torch.zeros(n_new, dtype=torch.int32, device="cuda")
        ok(lib.mi355_hyb_attention(out.data_ptr(), F32, Hh * d, 0, qn.data_ptr(), kp.data_ptr(), vp.data_ptr(), P(table, np.int32), P([L], np.int32),
                                   P([0, n_new], np.int32), tok_seq.data_ptr(), None, None, 1, n_new, Hh, G, d, d, bs, len(table), 1, chunk, 0, scale, 1.0, 0, 0,
                                   0.0, 0, dtype, _st()))
        got = out.cpu().numpy().reshape(n_new, Hh, d)
        assert np.abs(got - want).max() < tol(dtype, 5e-5, 3e-2) * max(1.0, np.abs(want).max()), pair


def test_chunk_of_one_token_is_the_token_itself_and_refusals(lib):
    _gpu()
    from candle_vllm_amd import hybrid_model as hm
    assert (hm.MASK_SLIDING, hm.MASK_CHUNKED) == (0, 1)
    x = dev(np.zeros((4, 8)))
    i = torch.zeros(8, dtype=torch.int32, device="cuda")

    def call(kind):
        return lib.mi355_hyb_attention(x.data_ptr(), F32, 8, 0, x.data_ptr(), x.data_ptr(), x.data_ptr(), i.data_ptr(), i.data_ptr(), i.data_ptr(), i.data_ptr(), None,
                                       None, 1, 1, 1, 1, 8, 8, 4, 1, kind, 4, 0, 1.0, 1.0, 0, 0, 0.0, 0, F32, _st())
    assert call(2) != 0 and call(-1) != 0
    assert lib.mi355_hyb_stream_step(x.data_ptr(), None, None, None, None, 0, None, None, None, None, None, None, F32, None, 1, 17, 8, 1e-5, _st()) != 0
    assert lib.mi355_hyb_decay_attention_scratch(256, 1, 4, 24, 32) == 0 and lib.mi355_hyb_decay_attention_scratch(256, 1, 4, 32, 48) == 5 * 4 * 32 * 48
    assert lib.mi355_hyb_decay_attention_scratch(63, 1, 4, 32, 32) == 0 and lib.mi355_hyb_decay_attention_scratch(300, 60, 4, 32, 32) == 0


@pytest.mark.parametrize("heads,d,vd,pieces", [(4, 24, 16, 0), (3, 5, 1, 0), (2, 64, 24, 0), (1, 200, 80, 0), (2, 400, 20, 0), (4, 32, 16, 1), (2, 16, 48, 1), (3, 128, 128, 1),
                                               (1, 256, 144, 1), (2, 48, 32, 1), (1, 512, 16, 1), (2, 64, 64, 1)])
def test_constant_decay_attention_over_portions_and_reused_slots(lib, heads, d, vd, pieces):
    """two unequal sequences side by side in portions (of 1, 2, 63, 64, 65, 190 ... tokens) that continue from their slots, as a scan and
    by pieces of 64 tokens on the matrix cores; decays 0 and 1 among them; stale slots (position 0 starts from zero), a slot used again"""
    _gpu()
    rng = np.random.default_rng(heads * 1000 + d)
    ld, stride, n_slots = heads * (2 * d + vd) + 4, heads * d * vd + 11, 3
    q_off, k_off, v_off = 4, 4 + heads * d, 4 + 2 * heads * d
    decay = f32(([0.6, 0.999, 0.0, 1.0] if d != 24 else [1.0, 0.93, 0.5, 0.9999])[:heads])
    state = dev(rng.standard_normal((n_slots, stride)))

    def make(T):
        x = f32(rng.standard_normal((T, ld)) / math.sqrt(math.sqrt(d)))
        o, Sf = S.decay_recurrence(x[:, q_off:k_off].reshape(T, heads, d), x[:, k_off:v_off].reshape(T, heads, d), x[:, v_off:].reshape(T, heads, vd), decay)
        return x, o, Sf

    def run(seqs):
        """seqs: [(rows, slot, context length behind the portion)]"""
        xs, cu = np.concatenate([s[0] for s in seqs]), np.cumsum([0] + [len(s[0]) for s in seqs])
        T = int(cu[-1])
        o = torch.zeros((T, heads, vd), device="cuda")
        scratch = torch.full(((T // 64 + len(seqs)) * heads * d * vd,), float("nan"), device="cuda")
        ok(lib.mi355_hyb_decay_attention(o.data_ptr(), state.data_ptr(), stride, P(xs), ld, q_off, k_off, v_off, P(decay), P([s[2] for s in seqs], np.int32),
                                         P(cu, np.int32), P([s[1] for s in seqs], np.int32), len(seqs), T, heads, d, vd, scratch.data_ptr() if pieces else None, _st()))
        return o.cpu().numpy()
    cutsA, cutsB = ([1, 2, 63, 64, 65, 190, 1], [3, 1, 1, 130, 0, 2, 64]) if pieces else ([1, 2, 9, 1, 27], [3, 1, 1, 12, 0])
    A, B = make(sum(cutsA)), make(sum(cutsB))
    la = lb = 0
    gotA, gotB = [], []
    for ca, cb in zip(cutsA, cutsB):
        seqs = [(A[0][la:la + ca], 2, la + ca)] + ([(B[0][lb:lb + cb], 0, lb + cb)] if cb else [])
        o = run(seqs)
        gotA.append(o[:ca]); gotB.append(o[ca:])
        la += ca; lb += cb
    for got, ref in ((np.concatenate(gotA), A), (np.concatenate(gotB), B)):
        assert np.abs(got - ref[1]).max() < 3e-5 * max(1.0, np.abs(ref[1]).max())
    st = state.cpu().numpy()
    for slot, ref in ((2, A), (0, B)):
        assert np.abs(st[slot, :heads * d * vd].reshape(heads, d, vd) - ref[2]).max() < 3e-5 * max(1.0, np.abs(ref[2]).max())
    C = make(70 if pieces else 6)                                          # a new sequence in A's slot: nothing of A is left
    assert np.abs(run([(C[0], 2, len(C[0]))]) - C[1]).max() < 3e-5 * max(1.0, np.abs(C[1]).max())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,n,groups", [(4, 64, 1), (3, 30, 3), (2, 1200, 1), (70, 300, 1), (5, 8, 8)])
def test_gate_behind_the_norm(lib, dtype, T, n, groups):
    _gpu()
    rng = np.random.default_rng(n)
    y, z, w = f32(3 * rng.standard_normal((T, n))), f32(rng.standard_normal((T, n + 5))), f32(1 + 0.2 * rng.standard_normal(n))
    out = empty_dt((T, n), dtype)
    ok(lib.mi355_hyb_norm_sigmoid_gate(out.data_ptr(), dtype, P(y), P(z), n + 5, P(w), T, n, groups, 1e-5, _st()))
    want = np.concatenate([S.norm_then_gate(p, ww, zz, 1e-5) for p, ww, zz in zip(np.split(y, groups, 1), np.split(w, groups), np.split(z[:, :n], groups, 1))], axis=1)
    assert np.abs(host_dt(out, dtype) - want).max() < tol(dtype, 2e-5, 8e-3) * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("T,W,E,top,append", [(9, 64, 16, 2, 0), (5, 50, 12, 3, 1), (7, 33, 70, 6, 1), (3, 128, 8, 8, 0), (6, 40, 1, 1, 1), (4, 64, 130, 5, 0), (300, 32, 9, 2, 1)])
def test_biased_router_softmax_over_the_chosen(lib, T, W, E, top, append):
    """z = router . h + bias in f32, the experts with the largest z, weights = softmax over those z alone; biases far apart must not flatten
    the choice among experts whose share of the whole softmax vanishes; the appended shared expert has weight 1"""
    _gpu()
    rng = np.random.default_rng(E * 10 + top)
    h, R, b = f32(rng.standard_normal((T, W))), f32(rng.standard_normal((E, W)) * 2 / math.sqrt(W)), f32(rng.standard_normal(E))
    if E > 2:
        b[1] = 150.0                                                      # exp(z - 150) is 0 in f32 for every other expert
    margins = []
    ids_w, w_w = S.route(h @ R.T + b, top, margins)
    ids = torch.zeros((T, top + append), dtype=torch.int32, device="cuda")
    wts = torch.zeros((T, top + append), device="cuda")
    ok(lib.mi355_hyb_moe_route_biased(ids.data_ptr(), wts.data_ptr(), None, None, F32, P(h), None, P(R), P(b), None, None, T, W, E, top, 1.0, 1e-5, append, 2, 0, 0, 1,
                                      _st()))
    sure = np.asarray(margins if margins else [np.inf] * T) > 1e-5
    assert sure.sum() >= T // 2
    assert np.array_equal(ids.cpu().numpy()[sure, :top], ids_w[sure])
    assert np.abs(wts.cpu().numpy()[sure, :top] - w_w[sure]).max() < 1e-5
    if append:
        assert (ids.cpu().numpy()[:, top] == E).all() and (wts.cpu().numpy()[:, top] == 1.0).all()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W,E,top,ff", [(5, 64, 6, 2, 24), (70, 64, 4, 3, 96), (200, 96, 3, 2, 64), (1, 32, 9, 9, 8)])
def test_grouped_relu2_experts(lib, dtype, T, W, E, top, ff):
    """grouping, the up product with relu^2 behind it, the down product and the weighted sum of the rows equal every expert run alone"""
    _gpu()
    rng = np.random.default_rng(T + E)
    h, up, dn = S.bf16_round(rng.standard_normal((T, W))), S.bf16_round(rng.standard_normal((E, ff, W)) / math.sqrt(W)), S.bf16_round(rng.standard_normal((E, W, ff)) / math.sqrt(ff))
    ids = np.stack([rng.permutation(E)[:top] for _ in range(T)])
    wt = f32(rng.uniform(0.1, 1, (T, top)))
    want = np.zeros((T, W))
    for t in range(T):
        for e, w in zip(ids[t], wt[t]):
            a = S.relu2(up[e] @ h[t])
            want[t] += w * (dn[e] @ (a if dtype == F32 else S.bf16_round(a)))
    pairs = T * top
    bm = min(lib.mi355_hyb_moe_block_rows(pairs, E, ff, W, dtype), lib.mi355_hyb_moe_block_rows(pairs, E, W, ff, dtype))
    nb = (pairs + bm - 1) // bm + E
    pos, tokrow, table = (torch.zeros(n, dtype=torch.int32, device="cuda") for n in (pairs, nb * bm, 2 * nb))
    ok(lib.mi355_hyb_moe_group(pos.data_ptr(), tokrow.data_ptr(), table.data_ptr(), P(ids, np.int32), pairs, top, E, bm, nb, _st()))
    act, y = empty_dt((nb * bm, ff), dtype), torch.zeros((nb * bm, W), device="cuda")
    ok(lib.mi355_hyb_linear_grouped_act(act.data_ptr(), dtype, ff, PD(h, dtype), dtype, W, tokrow.data_ptr(), PD(up, dtype), ff * W,
                                        table.data_ptr(), bm, nb, ff, W, 3, dtype, _st()))
    ok(lib.mi355_hyb_linear_grouped(y.data_ptr(), W, act.data_ptr(), dtype, ff, None, PD(dn, dtype), W * ff, table.data_ptr(), bm, nb, W, ff, dtype, _st()))
    got = (wt[:, :, None] * y.cpu().numpy()[pos.cpu().numpy().reshape(T, top)]).sum(1)
    assert np.abs(got - want).max() < tol(dtype, 2e-5, 2e-2) * max(1.0, np.abs(want).max())


# ------------------------------------------------------------------------------------------------------------ whole models
def _moe(E, top, ff, shared=None):
    m = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": E, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def _rot(dims, scaling=True):
    r = {"base": 3000.0, "dims": dims}
    if scaling:
        r["scaling"] = {"factor": 6.0, "fast": 16.0, "original": 64, "slow": 1.5}
    return r


def _att(heads, kv, dim, chunk, rot, scale=None):
    c = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": scale or 1.3 * dim ** -0.5, "vdim": dim}
    if rot:
        c["rot"] = rot
    if chunk:
        c["mask"] = {"size": chunk}
    return c


def _lin(heads, dim, vdim, decay=None):
    return {"decay": decay or [1.0 - 0.5 ** (1 + 2 * i) for i in range(heads)], "dim": dim, "heads": heads, "vdim": vdim}


def small_config(variant):
    dense = {"ff": 72, "kind": "dense"}
    if variant == 0:        # both mixers and feed-forwards, sizes that are not each other's equals, borrowed weights of both kinds of layer
        a, l = _att(4, 2, 16, 24, _rot(12), 0.9), _lin(3, 12, 20)
        layers = [{"type": "attention", "mixer": a, "mlp": _moe(7, 2, 24, 40)}, {"type": "lightning", "mixer": l, "mlp": dense},
                  {"type": "lightning", "mixer": l, "mlp": dense, "weights_of": 1}, {"type": "attention", "mixer": a, "mlp": _moe(7, 2, 24, 40), "weights_of": 0},
                  {"type": "lightning", "mixer": _lin(2, 32, 8), "mlp": None}]
        return {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": 61, "mul_cur": 5, "mul_prev": 23}, "scale": 3.0}, "layers": layers,
                "logit_softcap": 12.0, "norm": {"eps": 1e-5}, "streams": 3, "vocab": 131, "width": 64}
    if variant == 1:        # two streams, a shared expert of the experts' size, no shared expert, every expert chosen, no chunks, no rotation, no bigram
        layers = [{"type": "lightning", "mixer": _lin(2, 20, 12, [0.9, 1.0]), "mlp": _moe(5, 3, 32, 32)},
                  {"type": "attention", "mixer": _att(3, 3, 20, 0, _rot(20, False)), "mlp": _moe(4, 4, 24)},
                  {"type": "attention", "mixer": _att(6, 1, 8, 7, None, 0.5), "mlp": None}]
        return {"architecture": "Tosivik", "embedding": {"scale": 1.0}, "layers": layers, "norm": {"eps": 1e-6}, "streams": 2, "vocab": 90, "width": 100}
    if variant == 2:        # head sizes of the matrix-core kernels, pieces of the recurrence, prompts over several chunks
        layers = [{"type": "attention", "mixer": _att(8, 2, 64, 100, _rot(32), 0.3), "mlp": _moe(12, 3, 64, 96)},
                  {"type": "lightning", "mixer": _lin(4, 64, 32), "mlp": {"ff": 160, "kind": "dense"}},
                  {"type": "attention", "mixer": _att(2, 2, 32, 70, _rot(32)), "mlp": {"ff": 64, "kind": "dense"}},
                  {"type": "lightning", "mixer": _lin(2, 32, 64), "mlp": _moe(6, 1, 32, 32)}]
        return {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": 97, "mul_cur": 1, "mul_prev": 1}, "scale": 5.0}, "layers": layers,
                "logit_softcap": 25.0, "norm": {"eps": 1e-5}, "streams": 5, "vocab": 257, "width": 160}
    # no `streams`: the plain pre-norm form
    layers = [{"type": "attention", "mixer": _att(4, 1, 32, 40, _rot(16)), "mlp": dense}, {"type": "lightning", "mixer": _lin(1, 16, 16), "mlp": _moe(3, 1, 16, 16)}]
    return {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": 1, "mul_cur": 3, "mul_prev": 2}}, "layers": layers, "norm": {"eps": 1e-5}, "vocab": 64,
            "width": 48}


def weights(cfg, rng):
    """random weights; a configuration without `streams` has no mixing tensors: the oracle gets ones"""
    W = S.random_tosivik(rng, cfg)
    if not cfg.get("streams"):
        for k in W:
            if ".hc" in k:
                W[k] = np.ones_like(W[k])
    return W


def stored(cfg, W):
    return {k: v for k, v in W.items() if cfg.get("streams") or ".hc" not in k}


def settle_router(cfg, W, rng):
    """routing for runs in 16 bits: rounding noise flips a choice between two experts whose logits are close, and the oracle cannot follow
    such a flip.  A bias that lifts some experts of a layer far above the rest settles the choice; the weights among them still come
    from the router.  The choice by token is what the f32 runs cover."""
    for i, lc in enumerate(cfg["layers"]):
        k = "l%d.mlp.router.b" % i
        if k in W:
            b = 0.3 * rng.standard_normal(W[k].shape)
            b[rng.permutation(len(b))[:lc["mlp"]["router"]["top"]]] += 30.0
            W[k] = S.bf16_round(b)


def model_of(cfg, W, dtype, block_size=16, state_slots=4):
    from candle_vllm_amd.hybrid_model import HybridModel, TosivikSpec
    W = stored(cfg, W)
    m = HybridModel(TosivikSpec(cfg, {k: v.shape for k, v in W.items()}), dtype=dtype, block_size=block_size, state_slots=state_slots)
    m.load_state_dict_f32(W)
    return m


def build(cfg, dtype, seed=0, block_size=16, state_slots=4):
    rng = np.random.default_rng(seed)
    W = weights(cfg, rng)
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
    """the error allowed at every position.  In 16 bits the norm behind the recurrence multiplies the rounding of h at positions where
    its output is nearly zero (a token whose q . k is small): there, three times the largest of what five roundings of the sublayers'
    inputs (to nearest, and errors of up to half a last place at random) do to the oracle"""
    if dtype == "float32":
        return np.full(len(toks), TOL[dtype])
    rng = np.random.default_rng(0)

    def half_place(h):
        return h * (1.0 + rng.uniform(-1, 1, h.shape) / 512.0)
    noise = [row_errs(S.forward(cfg, W, toks, operand=f)[0], want) for f in [S.bf16_round] + [half_place] * 4]
    return np.maximum(TOL[dtype], 3.0 * np.max(noise, axis=0))


CLOSE_CALL = 1e-5           # a choice between two experts (or groups) whose scores lie closer than this may fall either way in f32


def oracle_logits(cfg, W, toks, rng=None):
    """the oracle's logits (and trace); no routing decision of the run may be a close call -- with `rng`, tokens are drawn again"""
    for _ in range(30):
        margins = []
        out, tr = S.forward(cfg, W, toks, margins)
        if not margins or min(margins) > CLOSE_CALL:
            return out, tr, toks
        assert rng is not None, "a routing decision of this test is a close call: take other tokens"
        toks = rng.integers(0, cfg["vocab"], len(toks)).tolist()
    raise AssertionError("no token sequence without a close call")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("variant", [0, 1, 2, 3])
def test_model_whole_portions_decode_against_oracle(lib, dtype, variant):
    """one request whole, with the residual stream behind every layer; then the same tokens in portions of 2, 1, 17, ... tokens and
    token by token: every way must give the oracle's logits at every position (the previous token, recurrent state and chunks
    cross every cut; pages of 16 tokens)"""
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
    want = {r: S.forward(cfg, W, toks[r])[0] for r in toks}
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
    """one head, one expert of which one is used, one stream with mixing weights of its own, head sizes of one, chunks of one token, one bucket"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    layers = [{"type": "lightning", "mixer": _lin(1, 1, 1), "mlp": _moe(1, 1, 8, 1)},
              {"type": "attention", "mixer": _att(1, 1, 1, 1, None), "mlp": {"ff": 1, "kind": "dense"}},
              {"type": "attention", "mixer": _att(2, 1, 2, 3, _rot(2)), "mlp": _moe(3, 3, 1, 1)}]
    cfg = {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": 1, "mul_cur": 1, "mul_prev": 1}, "scale": 2.0}, "layers": layers, "logit_softcap": 5.0,
           "norm": {"eps": 1e-5}, "streams": 1, "vocab": 17, "width": 32}
    m, W = build(cfg, "float32", seed=5)
    rng = np.random.default_rng(5)
    want, _, toks = oracle_logits(cfg, W, rng.integers(0, 17, 40).tolist(), rng)
    eng = StepEngine(m, 64)
    lo, rows = 0, []
    for c in [1, 2, 20, 1, 1, 15]:
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
            lg = S.forward(cfg, W, seq)[0][-1]
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
    W = weights(cfg, rng)
    if dtype == "bfloat16":
        settle_router(cfg, W, rng)
    _write_model(tmp_path, cfg, W)
    lens = {"a": 150, "b": 40, "c": 3, "d": 90, "e": 61, "f": 130}
    toks = {r: oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], n).tolist(), rng)[2] for r, n in lens.items()}
    want = {r: S.forward(cfg, W, toks[r])[0] for r in toks}
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
    """sizes, head counts, depth, order, streams, expert counts and constants drawn at random (sizes that are not all multiples of 16 or 32;
    layers without a feed-forward or a shared expert, borrowed weights)"""
    def mlp():
        u = rng.random()
        if u < 0.15:
            return None
        if u < 0.5:
            return {"ff": int(rng.choice([24, 100, 256])), "kind": "dense"}
        E, ff = int(rng.choice([2, 5, 16, 24])), int(rng.choice([16, 40, 64]))
        return _moe(E, int(rng.integers(1, min(E, 6) + 1)), ff, [None, ff, 48][int(rng.integers(0, 3))])
    layers = []
    for i in range(int(rng.integers(3, 7))):
        own = [j for j, lc in enumerate(layers) if "weights_of" not in lc]
        if own and rng.random() < 0.3:
            j = int(rng.choice(own))
            layers.append(dict(layers[j], weights_of=j))
            continue
        if rng.random() < 0.5:
            h = int(rng.choice([1, 2, 3, 4]))
            c = _lin(h, int(rng.choice([8, 16, 20, 32, 64, 128])), int(rng.choice([8, 16, 32, 48, 64, 100])), [float(x) for x in rng.uniform(0.3, 1.0, h)])
            layers.append({"type": "lightning", "mixer": c, "mlp": mlp()})
        else:
            G, d = int(rng.choice([1, 2, 3])), int(rng.choice([16, 20, 32, 48, 64, 128]))
            rot = None
            if rng.random() < 0.9:
                rot = {"base": float(rng.choice([1e3, 1e4, 5e5])), "dims": int(rng.choice([n for n in (2, 8, 16, d) if n <= d]))}
                if rng.random() < 0.8:
                    rot["scaling"] = {"factor": float(rng.choice([2.0, 8.0, 40.0])), "fast": float(rng.choice([8.0, 32.0])),
                                      "original": int(rng.choice([64, 1024, 4096])), "slow": float(rng.choice([0.5, 1.0, 2.0]))}
            c = _att(G * int(rng.choice([1, 2, 3, 4])), G, d, int(rng.choice([5, 32, 64, 77, 130])), rot, float(d ** -0.5 * rng.uniform(0.7, 2.0)))
            layers.append({"type": "attention", "mixer": c, "mlp": mlp()})
    cfg = {"architecture": "Tosivik", "embedding": {"scale": float(rng.choice([1.0, 4.0, 9.0]))}, "layers": layers, "logit_softcap": float(rng.choice([8.0, 20.0, 50.0])),
           "norm": {"eps": float(rng.choice([1e-5, 1e-6]))}, "streams": int(rng.choice([1, 2, 3, 6, 9])), "vocab": int(rng.integers(50, 600)),
           "width": int(rng.choice([64, 100, 128, 160, 256]))}
    if rng.random() < 0.8:
        cfg["embedding"]["bigram"] = {"buckets": int(rng.integers(1, 300)), "mul_cur": int(rng.integers(1, 200)), "mul_prev": int(rng.integers(1, 200))}
    return cfg


@pytest.mark.parametrize("seed", [2, 11, 21, 33, 47, 58])
def test_random_configurations_whole_and_mixed_schedules(lib, seed):
    """three unequal requests of a random configuration: each alone in one step, then together in a random schedule of portions (2, 3,
    17, 64, 65, 100 tokens; a request may sit a step out) that ends token by token -- on 64-token pages, in f32 and bf16"""
    _gpu()
    from candle_vllm_amd.step_engine import StepEngine
    rng = np.random.default_rng(seed)
    cfg = random_config(rng)
    W = weights(cfg, rng)
    lens = [int(rng.integers(150, 300)), int(rng.integers(1, 40)), int(rng.integers(60, 130))]
    toks = [oracle_logits(cfg, W, rng.integers(0, cfg["vocab"], n).tolist(), rng)[2] for n in lens]
    want = [S.forward(cfg, W, t)[0] for t in toks]
    for dtype in ("float32", "bfloat16"):
        if dtype == "bfloat16":
            settle_router(cfg, W, rng)
            want = [S.forward(cfg, W, t)[0] for t in toks]
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
