"""Host side of the Tosivik design, no GPU: config.json -> layer structs and weight slots (every size and constant from the config or a
tensor's shape, absent parts), the registry, the rotation tables against the oracle's angles, what the host layer refuses, and the
oracle's own invariants by hand (mixing of the streams, pairs of tokens, chunk edges, values that do not turn, the recurrence in portions,
the router's choice and weights)."""
import ctypes
import math

import numpy as np
import pytest

from oracle import tosivik as S


def _cfg():
    rot = {"base": 7000.0, "dims": 8, "scaling": {"factor": 3.0, "fast": 8.0, "original": 128, "slow": 0.5}}
    att = {"dim": 12, "heads": 6, "kv_heads": 3, "mask": {"size": 33}, "rot": rot, "scale": 0.3, "vdim": 12}
    lin = {"decay": [0.5, 0.25, 0.9990234375], "dim": 10, "heads": 3, "vdim": 14}
    moe = {"expert": {"ff": 9}, "kind": "moe", "router": {"experts": 5, "top": 2}, "shared": {"ff": 11}}
    moe2 = {"expert": {"ff": 7}, "kind": "moe", "router": {"experts": 4, "top": 1}, "shared": {"ff": 7}}
    free = {"dim": 12, "heads": 2, "kv_heads": 2, "scale": 0.2, "vdim": 12}
    return {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": 30, "mul_cur": 3, "mul_prev": 7}, "scale": 0.25},
            "layers": [{"type": "attention", "mixer": att, "mlp": moe}, {"type": "lightning", "mixer": lin, "mlp": {"ff": 21, "kind": "dense"}},
                       {"type": "attention", "mixer": att, "mlp": moe, "weights_of": 0}, {"type": "attention", "mixer": free, "mlp": None},
                       {"type": "lightning", "mixer": dict(lin, decay=[0.1, 0.2, 0.3]), "mlp": moe2}],
            "logit_softcap": 9.0, "norm": {"eps": 1e-6}, "streams": 3, "vocab": 77, "width": 40}


def _spec(cfg, W):
    from candle_vllm_amd import hybrid_model as hm
    return hm.TosivikSpec(cfg, {k: v.shape for k, v in W.items()})


def test_spec_reads_every_size_from_config_and_shapes(lib):
    from candle_vllm_amd import hybrid_model as hm
    cfg = _cfg()
    W = S.random_tosivik(np.random.default_rng(0), cfg)
    spec = _spec(cfg, W)
    a, b, c, d, e = spec.layers
    assert (spec.residual_form, spec.streams, spec.bigram_buckets, spec.bigram_mul_prev, spec.bigram_mul_cur) == (4, 3, 30, 7, 3)
    assert abs(spec.embed_scale - 0.25) < 1e-9 and abs(spec.logit_softcap - 9.0) < 1e-9 and abs(spec.eps - 1e-6) < 1e-12
    assert (a.mixer, a.a_heads, a.a_kv_heads, a.a_dim, a.a_vdim, a.a_rot_dims, a.a_rot_interleaved, a.a_window, a.a_mask_kind, a.a_v_is_k, a.share_with) == \
        (hm.MIX_ATTENTION, 6, 3, 12, 12, 8, 0, 33, hm.MASK_CHUNKED, 1, 0)
    assert (a.mlp_kind, a.mlp_ff, a.moe_experts, a.moe_top, a.moe_shared_ff, a.moe_relu2, a.moe_bias, a.moe_shared_plain) == (hm.MLP_MOE, 9, 5, 2, 11, 1, 1, 1)
    assert (b.mixer, b.d_heads, b.d_dim, b.d_vdim, b.mlp_kind, b.mlp_ff) == (hm.MIX_DECAY, 3, 10, 14, hm.MLP_GELU, 21)
    assert c.share_with == 1 and spec.slots[2] == {} and spec.rope[2] is None and spec.rope[0]["dims"] == 8
    assert (d.a_window, d.a_mask_kind, d.a_rot_dims, d.mlp_kind) == (0, hm.MASK_SLIDING, 0, 0) and spec.rope[3] is None
    offs = (ctypes.c_int32 * 9)()
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(a), offs) == 72 + 36 and list(offs)[:3] == [0, 72, 72]
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(b), offs) == 30 + 30 + 42 + 42 and (offs[3], offs[4], offs[5], offs[8]) == (0, 30, 60, 102)
    s0, s1, _, s3, s4 = spec.slots
    assert s0[hm.HW_IN_PROJ] == ["l0.mix.q", "l0.mix.k"] and s1[hm.HW_IN_PROJ] == ["l1.mix.q", "l1.mix.k", "l1.mix.v", "l1.mix.g"]
    assert np.array_equal(s1[hm.HW_D_DECAY][0].values, np.float32([0.5, 0.25, 0.9990234375]))
    assert s0[hm.HW_MLP_GATE_UP] == ["l0.mlp.shared.up"] and len(s0[hm.HW_MOE_GATE_UP]) == 5 and s0[hm.HW_MOE_BIAS] == ["l0.mlp.router.b"]
    assert hm.HW_MLP_GATE_UP not in s4 and s4[hm.HW_MOE_GATE_UP][-1] == "l4.mlp.shared.up"      # of the experts' size: one more group
    assert s3[hm.HW_HC1_MIX] == ["l3.hc1.mix"] and hm.HW_HC2_MIX not in s3 and hm.HW_NORM2 not in s3
    used = {n for sl in spec.slots for names in sl.values() for n in names if isinstance(n, str)} | set(spec.globals_().values())
    assert used == set(W)                                                    # every tensor of the checkpoint has a slot
    with pytest.raises(ValueError):
        _spec({**cfg, "layers": [{"type": "delta", "mixer": {}, "mlp": None}]}, W)
    with pytest.raises(ValueError):
        _spec({**cfg, "layers": [dict(cfg["layers"][1], mlp={"kind": "glu", "ff": 8})]}, W)
    with pytest.raises(ValueError):
        _spec({**cfg, "layers": [dict(cfg["layers"][0], weights_of=1), dict(cfg["layers"][0], weights_of=0)]}, W)


def test_absent_parts(lib):
    """no streams (the plain pre-norm form: one copy, every mixing weight 1), no bigram, no softcap, no scale, a chain of borrowed weights"""
    from candle_vllm_amd import hybrid_model as hm
    cfg = _cfg()
    del cfg["streams"], cfg["embedding"], cfg["logit_softcap"]
    cfg["layers"].append(dict(cfg["layers"][0], weights_of=2))
    W = {k: v for k, v in S.random_tosivik(np.random.default_rng(0), cfg).items() if ".hc" not in k}
    spec = _spec(cfg, W)
    assert (spec.streams, spec.bigram_buckets, spec.logit_softcap, spec.embed_scale) == (1, 0, 0.0, 1.0)
    assert hm.HW_BIGRAM not in spec.globals_() and spec.slots[0][hm.HW_HC2_MIX][0].n == 1
    assert spec.layers[5].share_with == 1                                    # the layer at the end of the chain


def test_registry_serves_the_design():
    from candle_vllm_amd import registry
    assert "Tosivik" in registry.registered()
    assert registry.component_of({"architecture": "Tosivik"}) == "hybrid"


@pytest.mark.parametrize("rot", [{"base": 10000.0, "dims": 32, "scaling": {"factor": 2.0, "fast": 32.0, "original": 1024, "slow": 1.0}},
                                 {"base": 500000.0, "dims": 128, "scaling": {"factor": 40.0, "fast": 16.0, "original": 4096, "slow": 2.0}},
                                 {"base": 1000.0, "dims": 6, "scaling": {"factor": 3.5, "fast": 8.0, "original": 64, "slow": 0.5}},
                                 {"base": 50.0, "dims": 8, "scaling": {"factor": 4.0, "fast": 32.0, "original": 16, "slow": 30.0}},
                                 {"base": 123456.0, "dims": 16, "scaling": {"factor": 1.0, "fast": 32.0, "original": 256, "slow": 1.0}},
                                 {"base": 7000.0, "dims": 24}])
def test_rotation_tables_follow_the_oracles_angles(lib, rot):
    from candle_vllm_amd.hybrid_model import TosivikSpec
    n, dims = 700, rot["dims"]
    rs = TosivikSpec.rope_scaling(rot)
    cos, sin = np.zeros((n, dims // 2), np.float32), np.zeros((n, dims // 2), np.float32)
    assert lib.mi355_rope_tables_f64(cos.ctypes.data, sin.ctypes.data, dims, n, float(rot["base"]), ctypes.byref(rs), n, n) == 0
    ang, amp = S.yarn_angles(rot, n)
    assert np.abs(cos - np.cos(ang) * amp).max() < 2e-6 and np.abs(sin - np.sin(ang) * amp).max() < 2e-6


def test_streams_and_pairs_of_tokens_by_hand():
    X = np.array([[[1.0, 2.0]], [[10.0, 20.0]]])
    M, b, y = np.array([[0.5, 3.0], [0.25, 0.0]]), np.array([1.0, -1.0]), np.array([[100.0, 200.0]])
    assert np.allclose(S.stream_mixture(X, np.array([2.0, 0.1])), [[3.0, 6.0]])
    assert np.allclose(S.stream_update(X, M, b, y), [[[0.5 + 2.5 + 100, 1 + 5 + 200]], [[3.0 - 100, 6.0 - 200]]])      # rows: from, columns: to
    assert S.bigram_rows([5, 9, 0, 5], 11, 7, 3) == [11, (35 + 27) % 11, 63 % 11, 15 % 11]


def test_chunk_edges_and_values_that_do_not_turn():
    m = S.chunk_mask(7, 3)
    assert m.sum(1).tolist() == [1, 2, 3, 1, 2, 3, 1] and m[5].tolist() == [False, False, False, True, True, True, False]
    assert S.chunk_mask(4, 0).sum() == 10 and S.chunk_mask(4, 1).sum() == 4
    q = k = np.zeros((4, 1, 2))
    v = np.arange(4.0).reshape(4, 1, 1)
    assert np.allclose(S.softmax_attention(q, k, v, 1.0, S.chunk_mask(4, 2))[:, 0, 0], [0, 0.5, 2, 2.5])
    # with scores that only depend on the distance, a turned value would show: the output is the unturned keys' mean
    cfg = {"dim": 4, "heads": 1, "kv_heads": 1, "rot": {"base": 10.0, "dims": 4}, "scale": 0.0, "vdim": 4}
    h = np.random.default_rng(0).standard_normal((3, 4))
    W = {"q": np.eye(4), "k": np.eye(4), "o": np.eye(4)}
    assert np.allclose(S.chunk_attention(h, W, "", cfg)[2], h.mean(0))
    x = np.random.default_rng(1).standard_normal((1, 1, 6))
    ang = np.array([[math.pi / 2, 0.0]])
    y = S.rotate_halves(x, ang, 2.0, 4)[0, 0]                                # dimension 0 turns with dimension 2, dimensions 4 and 5 pass
    assert np.allclose(y, [-2 * x[0, 0, 2], 2 * x[0, 0, 1], 2 * x[0, 0, 0], 2 * x[0, 0, 3], x[0, 0, 4], x[0, 0, 5]])


def test_recurrence_in_portions_by_pieces_and_by_hand():
    rng = np.random.default_rng(1)
    T, H, d, vd = 13, 3, 4, 5
    q, k, v, a = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, vd)), np.array([0.5, 1.0, 0.0])
    o, Sf = S.decay_recurrence(q, k, v, a)
    st, parts = None, []
    for lo, hi in ((0, 1), (1, 3), (3, 4), (4, 13)):
        op, st = S.decay_recurrence(q[lo:hi], k[lo:hi], v[lo:hi], a, st)
        parts.append(op)
    assert np.abs(np.concatenate(parts) - o).max() < 1e-12 and np.abs(st - Sf).max() < 1e-12
    for h in range(H):                                                       # o_t = sum_(u <= t) a^(t-u) (q_t . k_u) v_u
        p = np.tril(q[:, h] @ k[:, h].T) * np.where(np.tril(np.ones((T, T))) > 0, a[h] ** np.maximum(np.subtract.outer(np.arange(T), np.arange(T)), 0), 0)
        assert np.abs(p @ v[:, h] - o[:, h]).max() < 1e-12


def test_router_by_hand():
    z = np.log(np.array([[1.0, 4.0, 2.0, 3.0], [5.0, 1.0, 5.0, 1.0]]))
    ids, w = S.route(z, 2)
    assert ids.tolist() == [[1, 3], [0, 2]] and np.allclose(w, [[4 / 7, 3 / 7], [0.5, 0.5]])
    assert np.allclose(S.relu2(np.array([-2.0, 3.0])), [0.0, 9.0])


def test_host_layer_refuses_what_it_does_not_serve(lib):
    """create() checks what needs no device"""
    from candle_vllm_amd._lib import HybridConfig, HybridLayer
    cfg = _cfg()
    W = S.random_tosivik(np.random.default_rng(0), cfg)

    def create(mutate=lambda layers: None, **kw):
        spec = _spec(cfg, W)
        mutate(spec.layers)
        n = len(spec.layers)
        arr = (HybridLayer * n)(*spec.layers)
        c = dict(width=40, vocab=77, n_layers=n, dtype=0, block_size=16, state_slots=2, norm_eps=1e-6, unit_eps=1e-6, residual_form=4, resid_alpha=1.0,
                 norm_groups=1, logit_scale=1.0, norm_kind=0, embed_scale=0.25, logit_softcap=9.0, tie_head=0, side_cols=0, streams=3, bigram_buckets=30,
                 bigram_mul_prev=7, bigram_mul_cur=3)
        c.update(kw)
        h = lib.mi355_hybrid_create(ctypes.byref(HybridConfig(**c)), arr)
        if h:
            floats = lib.mi355_hybrid_state_floats_per_slot(h)
            lib.mi355_hybrid_destroy(h)
            return floats
        return None

    def set_(i, **kw):
        def f(layers):
            for k, v in kw.items():
                setattr(layers[i], k, v)
        return f
    assert create() == 2 * 3 * 10 * 14 + 1                                   # the states of both recurrences and the previous token
    assert create(bigram_buckets=0) == 2 * 3 * 10 * 14
    assert create(streams=0) is None and create(streams=17) is None and create(residual_form=3) is None and create(bigram_mul_prev=-1) is None
    assert create(width=12289) is None
    assert create(set_(0, a_vdim=8)) is None                                 # the values are the keys: one size
    assert create(set_(0, a_mask_kind=2)) is None
    assert create(set_(1, d_dim=513)) is None
    assert create(set_(1, a_v_is_k=1)) is None
    assert create(set_(2, a_window=32)) is None                              # borrowed weights, another shape
    assert create(set_(0, moe_relu2=0)) is None
    assert create(set_(1, moe_bias=1)) is None
