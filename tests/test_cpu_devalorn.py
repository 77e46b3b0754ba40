"""Host side of the Devalorn design, no GPU: config.json -> layer structs and weight slots (every size and constant from the config or a
tensor's shape, segments of the input projection, absent parts, borrowed keys and values), the registry, the rotation tables against the
oracle's angles, what the host layer refuses, and the oracle's own invariants by hand (mixtures of neighbouring tokens, the recurrence in
portions and by pieces, window edges and kept tokens, the distance bias, the query temperature, the router's weights)."""
import ctypes
import math

import numpy as np
import pytest

from oracle import devalorn as D


def _cfg():
    left = {"dim": 12, "heads": 6, "kv_heads": 3, "mask": {"keep_first": 4, "size": 33}, "rot": {"base": 7000.0, "dims": 8}, "scale": 0.3, "vdim": 20}
    par = {"left": left, "left_scale": 0.75, "right": {"dim": 10, "heads": 3}, "right_scale": 1.25}
    att = {"dim": 14, "heads": 4, "kv_heads": 2, "mask": {"size": 19}, "q_temp": {"coef": 0.25, "every": 12}, "scale": 0.2, "vdim": 6}
    moe = {"expert": {"ff": 9}, "kind": "moe", "router": {"experts": 5, "scale": 1.75, "top": 2}}
    return {"architecture": "Devalorn",
            "layers": [{"type": "attention", "mixer": att, "mlp": moe}, {"type": "parallel", "mixer": par, "mlp": {"ff": 21, "kind": "dense"}},
                       {"type": "attention", "mixer": dict(att, heads=8, kv_from=0, mask={"size": 7}), "mlp": None}],
            "norm": {"eps": 1e-6}, "vocab": 77, "width": 40}


def _weights(cfg, **kw):
    return D.random_devalorn(np.random.default_rng(0), cfg, **kw)


def _spec(cfg, W):
    from candle_vllm_amd import hybrid_model as hm
    return hm.DevalornSpec(cfg, {k: v.shape for k, v in W.items()})


def test_spec_reads_every_size_from_config_and_shapes(lib):
    from candle_vllm_amd import hybrid_model as hm
    cfg = _cfg()
    W = _weights(cfg, rank=7, right_vdim=11)
    spec = _spec(cfg, W)
    a, b, c = spec.layers
    assert spec.residual_form == 5 and abs(spec.eps - 1e-6) < 1e-12 and (spec.width, spec.vocab) == (40, 77)
    assert (a.mixer, a.a_heads, a.a_kv_heads, a.a_dim, a.a_vdim, a.a_window, a.a_keep_first, a.a_rot_dims, a.a_qk_norm, a.a_norm_whole, a.a_dist_bias, a.a_head_gate,
            a.kv_from) == (hm.MIX_ATTENTION, 4, 2, 14, 6, 19, 0, 0, 1, 1, hm.DIST_LINEAR, 0, 0)
    assert abs(a.a_temp_coef - 0.25) < 1e-7 and a.a_temp_every == 12.0 and abs(a.a_scale - 0.2) < 1e-7
    assert (a.mlp_kind, a.mlp_ff, a.moe_experts, a.moe_top, a.moe_shared_ff, a.moe_normalise) == (hm.MLP_MOE, 9, 5, 2, 0, 0) and abs(a.moe_scale - 1.75) < 1e-7
    assert (b.mixer, b.a_heads, b.a_kv_heads, b.a_dim, b.a_vdim, b.a_window, b.a_keep_first, b.a_rot_dims, b.a_rot_interleaved, b.a_qk_norm, b.a_dist_bias,
            b.a_head_gate) == (hm.MIX_PARALLEL_TIMEMIX, 6, 3, 12, 20, 33, 4, 8, 0, 0, 0, 1)
    assert (b.d_heads, b.d_dim, b.d_vdim, b.d_a_rank, b.mlp_kind, b.mlp_ff) == (3, 10, 11, 7, hm.MLP_SILU_GLU, 21)
    assert abs(b.a_out_scale - 0.75) < 1e-7 and abs(b.d_out_scale - 1.25) < 1e-7 and b.a_temp_coef == 0.0 and spec.rope[1]["dims"] == 8
    assert (c.kv_from, c.a_window, c.mlp_kind, c.a_heads) == (1, 7, 0, 8)
    s0, s1, s2 = spec.slots
    d0 = s0[hm.HW_A_DIST][0].values
    assert np.allclose(d0, [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8] + [0] * 4)
    assert s0[hm.HW_IN_PROJ] == ["l0.mix.q", "l0.mix.k", "l0.mix.v"] and s2[hm.HW_IN_PROJ] == ["l2.mix.q"] and hm.HW_A_KNORM not in s2 and hm.HW_NORM2 not in s2
    # the projection of the parallel layer: whole 128-row tiles per segment, zeros behind the rows
    offs = (ctypes.c_int32 * 9)()
    att_rows = 72 + 36 + 60 + 6
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(b), offs) == 256 + 5 * 128
    assert list(offs) == [0, 72, 108, 256, 384, 512, 640, 768, 168]
    rows = [(n.rows if isinstance(n, hm.ZeroRows) else W[n].shape[0]) for n in s1[hm.HW_IN_PROJ]]
    assert rows == [72, 36, 60, 6, 256 - att_rows, 30, 98, 30, 98, 33, 95, 33, 95, 7, 121]
    assert [n for n in s1[hm.HW_IN_PROJ] if isinstance(n, str)] == ["l1.mix.left." + n for n in "qkvg"] + ["l1.mix.right." + n for n in ("r", "k", "v", "g", "w1")]
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(a), offs) == 56 + 28 + 12 and list(offs)[:3] == [0, 56, 84]
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(c), offs) == 112 and list(offs)[:3] == [0, -1, -1]
    t = s1[hm.HW_T_W2][0]
    assert np.array_equal(t.bits({"l1.mix.right.w2": np.arange(210, dtype=np.uint16)}, {"l1.mix.right.w2": (30, 7)}).reshape(7, 30), np.arange(210).reshape(30, 7).T)
    used = {getattr(n, "name", n) for sl in spec.slots for names in sl.values() for n in names if not isinstance(n, (hm.Constants, hm.ZeroRows))} | {"embed", "final.norm", "head"}
    assert used == set(W)                                                    # every tensor of the checkpoint has a slot
    for bad in ({"type": "delta", "mixer": {}, "mlp": None}, dict(cfg["layers"][1], mlp={"kind": "glu", "ff": 8})):
        with pytest.raises(ValueError):
            _spec({**cfg, "layers": [cfg["layers"][0], bad]}, W)
    with pytest.raises(ValueError):
        _spec({**cfg, "architecture": "Other"}, W)


def test_absent_parts(lib):
    """no windows, no kept tokens, no rotation, no temperature, no gate tensor, no router scale"""
    from candle_vllm_amd import hybrid_model as hm
    cfg = _cfg()
    for lc in cfg["layers"]:
        for m in (lc["mixer"], lc["mixer"].get("left", {})):
            for k in ("mask", "q_temp", "rot"):
                m.pop(k, None)
    del cfg["layers"][0]["mlp"]["router"]["scale"]
    W = {k: v for k, v in _weights(cfg).items() if not k.endswith("left.g")}
    a, b, c = _spec(cfg, W).layers
    assert (a.a_window, a.a_temp_coef, a.moe_scale, b.a_window, b.a_keep_first, b.a_rot_dims, b.a_head_gate, c.a_window) == (0, 0.0, 1.0, 0, 0, 0, 0, 0)
    assert "l1.mix.left.g" not in _spec(cfg, W).slots[1][hm.HW_IN_PROJ]
    assert lib.mi355_hybrid_in_proj_rows(ctypes.byref(b), None) == 256 + 5 * 128


def test_registry_serves_the_design():
    from candle_vllm_amd import registry
    assert "Devalorn" in registry.registered()
    assert registry.component_of({"architecture": "Devalorn"}) == "hybrid"


@pytest.mark.parametrize("rot", [{"base": 10000.0, "dims": 32}, {"base": 500000.0, "dims": 128}, {"base": 50.0, "dims": 6}, {"base": 1234.5, "dims": 2}])
def test_rotation_tables_follow_the_oracles_angles(lib, rot):
    from candle_vllm_amd.hybrid_model import DevalornSpec
    n, dims = 700, rot["dims"]
    half = dims // 2
    rs = DevalornSpec.rope_scaling(rot)
    cos, sin = np.zeros((n, half), np.float32), np.zeros((n, half), np.float32)
    assert lib.mi355_rope_tables_f64(cos.ctypes.data, sin.ctypes.data, dims, n, float(rot["base"]), ctypes.byref(rs), n, n) == 0
    x = np.zeros((n, 1, dims))
    x[:, 0, :half] = 1.0                                                     # u = 1, v = 0 turns into (cos, sin)
    y = D.rotate_halves(x, rot["base"], dims)[:, 0]
    assert np.abs(cos - y[:, :half]).max() < 2e-6 and np.abs(sin - y[:, half:]).max() < 2e-6


def test_mixtures_of_neighbouring_tokens_by_hand():
    h, mu = np.array([[1.0, 10.0], [3.0, 30.0]]), np.array([[0.0, 1.0], [0.5, 0.25]])
    assert np.allclose(D.token_mixes(h, mu), [[[1, 0], [3, 10]], [[0.5, 7.5], [2, 25]]])
    assert np.allclose(D.token_mixes(h[1:], mu, before=h[0]), D.token_mixes(h, mu)[:, 1:])


def test_recurrence_in_portions_by_pieces_and_by_hand():
    rng = np.random.default_rng(1)
    T, H, d, vd = 13, 2, 4, 5
    r, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, vd))
    w, u = rng.uniform(0, 1, (T, H, d)), rng.standard_normal((H, d))
    w[:, 0, 0], w[:, 1, 1] = 0.0, 1.0
    o, Sf = D.bonus_recurrence(r, k, v, w, u)
    st, parts = None, []
    for lo, hi in ((0, 1), (1, 3), (3, 4), (4, 13)):
        op, st = D.bonus_recurrence(r[lo:hi], k[lo:hi], v[lo:hi], w[lo:hi], u, st)
        parts.append(op)
    assert np.abs(np.concatenate(parts) - o).max() < 1e-12 and np.abs(st - Sf).max() < 1e-12
    for h in range(H):          # o_t = sum_(s < t) sum_i r_ti k_si prod_(s < a < t) w_ai v_s + (r_t . (u k_t)) v_t
        for t in range(T):
            e = (r[t, h] * u[h]) @ k[t, h] * v[t, h]
            for s in range(t):
                e = e + (r[t, h] * k[s, h] * np.prod(w[s + 1:t, h], axis=0)).sum() * v[s, h]
            assert np.abs(e - o[t, h]).max() < 1e-11
    # the same by pieces of 8 and sub-pieces of 4: only products of decays
    for h in range(H):
        S = np.zeros((d, vd))
        for lo in range(0, T, 8):
            hi = min(lo + 8, T)
            for t in range(lo, hi):
                b = lo + (t - lo) // 4 * 4
                rd = r[t, h] * np.prod(w[b:t, h], axis=0)
                e = (rd * np.prod(w[lo:b, h], axis=0)) @ S + (r[t, h] * u[h]) @ k[t, h] * v[t, h]
                for s in range(lo, t):
                    sb = lo + (s - lo) // 4 * 4
                    if sb == b:
                        e = e + (r[t, h] * k[s, h] * np.prod(w[s + 1:t, h], axis=0)).sum() * v[s, h]
                    else:
                        kd = k[s, h] * np.prod(w[s + 1:sb + 4, h], axis=0)
                        e = e + (rd * np.prod(w[sb + 4:b, h], axis=0)) @ kd * v[s, h]
                assert np.abs(e - o[t, h]).max() < 1e-11
            S = np.prod(w[lo:hi, h], axis=0)[:, None] * S + sum((k[s, h] * np.prod(w[s + 1:hi, h], axis=0))[:, None] * v[s, h] for s in range(lo, hi))
        assert np.abs(S - Sf[h]).max() < 1e-11
    assert np.allclose(D.lowrank_decay(np.zeros((1, 3)), np.ones((2, 3)), np.ones((4, 2)), np.array([0.0, 1.0, -50.0, 50.0])), [[math.exp(-1), math.exp(-math.e), 1, 0]])


def test_windows_kept_tokens_bias_and_temperature_by_hand():
    m = D.window_mask(7, 3, 2)
    assert m[5].tolist() == [True, True, False, True, True, True, False] and m.sum(1).tolist() == [1, 2, 3, 4, 5, 5, 5]
    assert D.window_mask(4, 0, 9).sum() == 10 and D.window_mask(4, 1).sum() == 4 and D.window_mask(5, 2).sum() == 9
    assert np.allclose(D.distance_slopes(2), [2.0 ** -4, 2.0 ** -8]) and np.allclose(D.distance_slopes(3)[0], 2.0 ** (-8 / 3))
    q = k = np.zeros((3, 1, 2))
    v = np.array([1.0, 2.0, 4.0]).reshape(3, 1, 1)
    o = D.grouped_attention(q, k, v, 1.0, D.window_mask(3, 2), np.array([math.log(3.0)]))[:, 0, 0]
    assert np.allclose(o, [1, (2 * 3 + 1) / 4, (4 * 3 + 2) / 4])
    t = D.query_temperature(9, 0.5, 4)
    assert np.allclose(t[[0, 2, 3, 6, 7]], [1, 1, 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(3)])
    assert np.allclose(D.head_norm_gate(np.array([[[3.0, 4.0], [0.0, 2.0]]]), np.array([1.0, 1, 2, 2]), 0.5, 0.0), [[3 / 12.5 ** 0.5 / 2, 4 / 12.5 ** 0.5 / 2, 0, 2 ** 0.5]])


def test_router_by_hand():
    z = np.log(np.array([[1.0, 4.0, 2.0, 3.0], [5.0, 1.0, 5.0, 1.0]]))
    ids, w = D.route(z, 2, 2.0)
    assert ids.tolist() == [[1, 3], [0, 2]] and np.allclose(w, [[0.8, 0.6], [10 / 12, 10 / 12]])       # not renormalised over the chosen ones


def test_host_layer_refuses_what_it_does_not_serve(lib):
    """create() checks what needs no device"""
    from candle_vllm_amd._lib import HybridConfig, HybridLayer
    cfg = _cfg()
    W = _weights(cfg)

    def create(mutate=lambda layers: None, **kw):
        spec = _spec(cfg, W)
        mutate(spec.layers)
        n = len(spec.layers)
        arr = (HybridLayer * n)(*spec.layers)
        c = dict(width=40, vocab=77, n_layers=n, dtype=0, block_size=16, state_slots=2, norm_eps=1e-6, unit_eps=1e-6, residual_form=5, resid_alpha=1.0,
                 norm_groups=1, logit_scale=1.0)
        c.update(kw)
        h = lib.mi355_hybrid_create(ctypes.byref(HybridConfig(**c)), arr)
        if h:
            out = (lib.mi355_hybrid_state_floats_per_slot(h), lib.mi355_hybrid_cache_bytes(h, 3))
            lib.mi355_hybrid_destroy(h)
            return out
        return None

    def set_(i, **kw):
        def f(layers):
            for k, v in kw.items():
                setattr(layers[i], k, v)
        return f
    floats = 3 * 10 * 10 + 40                                                # the recurrence's state and the last token's h
    pages = 3 * 16 * (2 * (14 + 6) + 3 * (12 + 20)) * 4                      # the borrowing layer holds no pages
    assert create() == (floats, floats * 4 * 2 + pages)
    assert create(residual_form=3) is None and create(residual_form=0) is None and create(norm_groups=2) is None and create(width=16385) is None
    assert create(set_(1, d_dim=513)) is None and create(set_(1, d_a_rank=0)) is None
    assert create(set_(0, a_temp_every=0.0)) is None
    assert create(set_(0, a_rot_dims=4)) is None                             # the norm over the whole projection does not rotate
    assert create(set_(0, a_dist_bias=3)) is None
    assert create(set_(2, kv_from=3)) is None and create(set_(2, a_dim=12)) is None and create(set_(2, kv_from=2)) is None    # a lender: earlier, same heads and sizes
    assert create(set_(0, moe_shared_ff=8)) is None
    assert create(set_(1, in_conv=3)) is None
    assert create(set_(1, mlp_kind=1)) is None
