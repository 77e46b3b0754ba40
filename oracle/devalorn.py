"""Slow float64 oracle of the Devalorn design, one function per mechanism, written from the equations and sharing nothing with
candle_vllm_amd/ or csrc/.  Test infrastructure only.  Whole sequences only (no cache; the recurrences can be given a starting state:
position t of a causal model is the truth for every way of cutting the sequence into steps).

The design: a layer-list decoder whose two sublayers read the same residual x through a norm of their own,
    x <- x + mixer(RMSnorm(x) w1) + ff(RMSnorm(x) w2).
Mixers: `attention` -- grouped heads, one RMS norm over the whole q and k projections, a query temperature that grows with the logarithm
of the position, a linear distance bias per head, a sliding window, optionally on an earlier layer's cached keys and values -- and
`parallel`: windowed attention with kept first tokens, rotate-half pairs and one sigmoid gate per head on the left, time mixing on the
right (every projection reads its own mixture of a token and the one before it; a matrix state per head with a decay per key channel
made from the token by a low-rank map, and a bonus for the current token), the two outputs scaled and added.  Feed-forward: silu
gate/up, or a mixture of such experts weighted by scaled softmax values.  Logits of a table of their own.

A model is (cfg, W): cfg the parsed config.json, W a dict name -> float64 ndarray."""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rotate_halves(x, base, dims):
    """x [T, heads, n], position = row: dimension i turns with dimension i + dims / 2, the dimensions from `dims` on pass"""
    if not dims:
        return x
    half = dims // 2
    f = float(base) ** (-2.0 * np.arange(half, dtype=np.float64) / dims)
    a = np.arange(x.shape[0], dtype=np.float64)[:, None, None] * f
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., dims:]], axis=-1)


def window_mask(T, size, keep=0):
    """[T, T] bool: query i sees key j <= i when i - j < size or j < keep (size 0: every earlier key)"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    m = j <= i
    return m & ((i - j < size) | (j < keep)) if size else m


def query_temperature(T, coef, every):
    return 1.0 + coef * np.log(np.floor((np.arange(T, dtype=np.float64) + 1.0) / every) + 1.0)


def distance_slopes(H):
    return 2.0 ** (-8.0 * (np.arange(H, dtype=np.float64) + 1.0) / H)


def grouped_attention(q, k, v, scale, mask, slopes=None):
    """q [T, H, d], k [T, G, d], v [T, G, vd] -> [T, H, vd]; slopes [H]: score - slope (i - j)"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if slopes is not None:
            s = s - slopes[h] * dist
        s = np.where(mask, s, -np.inf)
        e = np.exp(s - s.max(-1, keepdims=True))
        out[:, h] = (e / e.sum(-1, keepdims=True)) @ v[:, h // per]
    return out


def gated_window_attention(h, W, p, c):
    """the left branch, up to its output projection"""
    T, H, G, d, vd = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    rot, mask = c.get("rot") or {}, c.get("mask") or {}
    q = rotate_halves((h @ W[p + "q"].T).reshape(T, H, d), rot.get("base", 1.0), int(rot.get("dims", 0)))
    k = rotate_halves((h @ W[p + "k"].T).reshape(T, G, d), rot.get("base", 1.0), int(rot.get("dims", 0)))
    v = (h @ W[p + "v"].T).reshape(T, G, vd)
    o = grouped_attention(q, k, v, c["scale"], window_mask(T, int(mask.get("size", 0)), int(mask.get("keep_first", 0))))
    if p + "g" in W:
        o = o * sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * vd)


def previous_rows(h, before=None):
    """row t of the result is row t - 1 of h; row 0 is `before` (zeros at a sequence's start)"""
    first = np.zeros((1, h.shape[1])) if before is None else np.asarray(before, np.float64)[None]
    return np.concatenate([first, h[:-1]])


def token_mixes(h, mu, before=None):
    """mu [n, width] -> [n, T, width]: h + (previous h - h) mu_s"""
    back = previous_rows(h, before)
    return np.stack([h + (back - h) * m for m in mu])


def lowrank_decay(x, w1, w2, w0):
    """exp(-exp(W_2 tanh(W_1 x) + w_0)), per channel"""
    return np.exp(-np.exp(np.tanh(x @ w1.T) @ w2.T + w0))


def bonus_recurrence(r, k, v, w, u, S=None):
    """r, k, w [T, H, d], v [T, H, vd], u [H, d]: o_t = (S + diag(u) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T -> (o, S)"""
    T, H, d = r.shape
    S = np.zeros((H, d, v.shape[2])) if S is None else np.array(S, np.float64)
    o = np.zeros(v.shape)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S + u[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return o, S


def head_norm_gate(o, w, gate, eps):
    """o [T, H, vd] each head over its root mean square, then all heads side by side times w times the gate"""
    return unit_rms(o, eps).reshape(o.shape[0], -1) * w * gate


def time_mixing(h, W, p, c, eps):
    """the right branch, up to its output projection"""
    T, H, d = h.shape[0], c["heads"], c["dim"]
    xr, xk, xv, xg, xw = token_mixes(h, [W[p + "mu." + n] for n in "rkvgw"])
    r, k, v = ((x @ W[p + n].T).reshape(T, H, -1) for x, n in ((xr, "r"), (xk, "k"), (xv, "v")))
    w = lowrank_decay(xw, W[p + "w1"], W[p + "w2"], W[p + "w0"]).reshape(T, H, d)
    o, _ = bonus_recurrence(r, k, v, w, W[p + "u"].reshape(H, d))
    return head_norm_gate(o, W[p + "norm"], silu(xg @ W[p + "g"].T), eps)


def parallel_mixer(h, W, p, c, eps):
    left = gated_window_attention(h, W, p + "left.", c["left"]) @ W[p + "left.o"].T
    right = time_mixing(h, W, p + "right.", c["right"], eps) @ W[p + "right.o"].T
    return c["left_scale"] * left + c["right_scale"] * right


def whole_norm_keys(h, W, p, c, eps):
    """what an `attention` layer caches: keys behind their norm, values"""
    T, G = h.shape[0], c["kv_heads"]
    return ((unit_rms(h @ W[p + "k"].T, eps) * W[p + "k.norm"]).reshape(T, G, c["dim"]), (h @ W[p + "v"].T).reshape(T, G, c["vdim"]))


def biased_window_attention(h, W, p, c, kv, eps):
    T, H = h.shape[0], c["heads"]
    q = (unit_rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]).reshape(T, H, c["dim"])
    qt = c.get("q_temp")
    if qt:
        q = q * query_temperature(T, qt["coef"], qt["every"])[:, None, None]
    o = grouped_attention(q, kv[0], kv[1], c["scale"], window_mask(T, int((c.get("mask") or {}).get("size", 0))), distance_slopes(H))
    return o.reshape(T, H * c["vdim"]) @ W[p + "o"].T


def glu(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z, top, scale, margins=None):
    """z [T, E] -> the `top` experts with the largest softmax values (largest first, ties to the lower expert) and those values times
    scale.  margins: a list that receives, per token, by how much the last chosen logit beat the next"""
    ids = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    if margins is not None and top < z.shape[1]:
        s = -np.sort(-z, axis=-1)
        margins.extend((s[:, top - 1] - s[:, top]).tolist())
    e = np.exp(z - z.max(-1, keepdims=True))
    return ids, np.take_along_axis(e / e.sum(-1, keepdims=True), ids, axis=-1) * scale


def moe_ff(h, W, p, m, margins=None):
    ids, w = route(h @ W[p + "router"].T, m["router"]["top"], m["router"].get("scale", 1.0), margins)
    out = np.zeros((h.shape[0], W[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], w[t]):
            out[t] += wt * glu(h[t], W, p + "e%d." % e)
    return out


def forward(cfg, W, tokens, margins=None, operand=None):
    """-> logits [T, vocab], the residual behind every layer [n_layers, T, width]; margins: see route(); operand: what is done to every
    sublayer's normed input (a rounding: how far it alone moves the logits)"""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][np.asarray(tokens, np.int64)]
    cached, trace = {}, []
    for i, lc in enumerate(cfg["layers"]):
        p, c, m = "l%d." % i, lc["mixer"], lc.get("mlp")
        h = unit_rms(x, eps) * W[p + "norm1"]
        h = operand(h) if operand else h
        if lc["type"] == "parallel":
            y = parallel_mixer(h, W, p + "mix.", c, eps)
        else:
            cached[i] = whole_norm_keys(h, W, p + "mix.", c, eps) if c.get("kv_from") is None else cached[c["kv_from"]]
            y = biased_window_attention(h, W, p + "mix.", c, cached[i], eps)
        if m:
            h2 = unit_rms(x, eps) * W[p + "norm2"]
            h2 = operand(h2) if operand else h2
            y = y + (glu(h2, W, p + "mlp.") if m["kind"] == "dense" else moe_ff(h2, W, p + "mlp.", m, margins))
        x = x + y
        trace.append(x)
    return (unit_rms(x, eps) * W["final.norm"]) @ W["head"].T, np.stack(trace)


# ---------------------------------------------------------------------------------------------------------------- weights for tests
def bf16_round(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    r = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint32) << 16
    return r.view(np.float32).astype(np.float64)


def random_devalorn(rng, cfg, rank=6, right_vdim=None):
    """random bf16-representable weights for a config (f64 arrays): projections ~ N(0, 1/in), norms near 1, decays from nearly none to
    a tenth per token, mixtures that take anything from none to all of the token before"""
    W = {}

    def mat(name, rows, cols, s=None):
        W[name] = bf16_round(rng.standard_normal((rows, cols)) * (s if s is not None else 1.0 / math.sqrt(cols)))

    def vec(name, n, mean=0.0, s=0.1):
        W[name] = bf16_round(mean + s * rng.standard_normal(n))

    def attention(q, c):
        H, G, d, vd = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
        mat(q + "q", H * d, Wd)
        if c.get("kv_from") is None:
            mat(q + "k", G * d, Wd); mat(q + "v", G * vd, Wd)
        mat(q + "o", Wd, H * vd)

    Wd, V = cfg["width"], cfg["vocab"]
    mat("embed", V, Wd, 1.0)
    vec("final.norm", Wd, 1.0)
    mat("head", V, Wd, 2.0 / math.sqrt(Wd))
    for i, lc in enumerate(cfg["layers"]):
        p, c, m = "l%d." % i, lc["mixer"], lc.get("mlp")
        vec(p + "norm1", Wd, 1.0)
        if lc["type"] == "parallel":
            attention(p + "mix.left.", c["left"])
            mat(p + "mix.left.g", c["left"]["heads"], Wd, 2.0 / math.sqrt(Wd))
            q, H, d = p + "mix.right.", c["right"]["heads"], c["right"]["dim"]
            vd = right_vdim or d
            for n in "rkvgw":
                W[q + "mu." + n] = bf16_round(rng.uniform(0, 1, Wd))
            mat(q + "r", H * d, Wd); mat(q + "k", H * d, Wd); mat(q + "v", H * vd, Wd); mat(q + "g", H * vd, Wd)
            mat(q + "w1", rank, Wd); mat(q + "w2", H * d, rank)
            W[q + "w0"] = bf16_round(rng.uniform(-6, 1, H * d))
            vec(q + "u", (H, d), 0.3, 0.5); vec(q + "norm", H * vd, 1.0); mat(q + "o", Wd, H * vd)
        else:
            attention(p + "mix.", c)
            vec(p + "mix.q.norm", c["heads"] * c["dim"], 1.0, 0.2)
            if c.get("kv_from") is None:
                vec(p + "mix.k.norm", c["kv_heads"] * c["dim"], 1.0, 0.2)
        if not m:
            continue
        vec(p + "norm2", Wd, 1.0)
        for e in ([""] if m["kind"] == "dense" else ["e%d." % e for e in range(m["router"]["experts"])]):
            ff = m["ff"] if m["kind"] == "dense" else m["expert"]["ff"]
            mat(p + "mlp." + e + "gate", ff, Wd); mat(p + "mlp." + e + "up", ff, Wd); mat(p + "mlp." + e + "down", Wd, ff)
        if m["kind"] == "moe":
            mat(p + "mlp.router", m["router"]["experts"], Wd, 2.0 / math.sqrt(Wd))
    return W
