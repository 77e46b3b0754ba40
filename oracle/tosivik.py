"""Slow float64 oracle of the Tosivik design, one function per mechanism, written from the equations and sharing nothing with
candle_vllm_amd/ or csrc/.  Test infrastructure only.  Whole sequences only (no cache, no state: position t of a causal model is
the truth for every way of cutting the sequence into steps).

The design: a layer-list decoder whose residual stream is carried in s copies.  A sublayer f (mixer, then feed-forward) with weights
a [s], b [s], M [s, s] reads one mixture of the copies and writes to all of them,
    y = f(RMSnorm(sum_i a_i X_i) w),      X_j <- sum_i M[i, j] X_i + b_j y,
and the model's output is the sum of the copies.  Embedding: scaled token row + a row of a second table picked by a hash of (previous
token, token).  Mixers: grouped attention inside fixed chunks of positions whose values are the unrotated keys (rotate-half pairs, yarn
scaling), and linear attention with one constant decay per head behind a norm over all heads and a sigmoid gate.  Feed-forward: gelu
without a gate, or relu^2 experts chosen by biased logits (softmax over the chosen ones only) beside a shared expert of every token.
Logits of a table of their own, tanh-capped.

A model is (cfg, W): cfg the parsed config.json, W a dict name -> float64 ndarray."""
import math

import numpy as np


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """row of the second table for every token: (previous mul_prev + current mul_cur) mod buckets, the extra last row at the start"""
    return [buckets if t == 0 else (int(tokens[t - 1]) * mul_prev + int(tokens[t]) * mul_cur) % buckets for t in range(len(tokens))]


def embedding(cfg, W, tokens):
    e = cfg.get("embedding") or {}
    x = W["embed"][tokens] * float(e.get("scale", 1.0))
    b = e.get("bigram")
    return x + W["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])] if b else x


def stream_mixture(X, a):
    """X [s, T, width], a [s]"""
    return sum(a[i] * X[i] for i in range(X.shape[0]))


def stream_update(X, M, b, y):
    """M[i, j]: from copy i to copy j; b[j]: how much of the sublayer's output copy j takes"""
    s = X.shape[0]
    return np.stack([sum(M[i, j] * X[i] for i in range(s)) + b[j] * y for j in range(s)])


def yarn_angles(rot, T):
    """[T, dims / 2] angles and the amplitude on cos and sin"""
    dims, base = int(rot["dims"]), float(rot["base"])
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    amp = 1.0
    sc = rot.get("scaling")
    if sc:
        def at(turns):
            return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
        lo = max(math.floor(at(sc["fast"])), 0)
        hi = min(math.ceil(at(sc["slow"])), dims - 1)
        ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
        f = f / sc["factor"] * ramp + f * (1.0 - ramp)
        amp = 0.1 * math.log(sc["factor"]) + 1.0
    return np.arange(T, dtype=np.float64)[:, None] * f[None, :], amp


def rotate_halves(x, ang, amp, dims):
    """x [T, heads, n]: dimension i turns with dimension i + dims / 2, the dimensions from `dims` on pass"""
    half = dims // 2
    cos, sin = np.cos(ang)[:, None, :] * amp, np.sin(ang)[:, None, :] * amp
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], axis=-1)


def chunk_mask(T, size):
    """[T, T] bool: query i sees key j <= i of its own chunk of `size` positions (size 0: every earlier key)"""
    i = np.arange(T)
    m = i[:, None] >= i[None, :]
    return m & (i[:, None] // size == i[None, :] // size) if size else m


def softmax_attention(q, k, v, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, vd] -> [T, H, vd]"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(mask, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        e = np.exp(s - s.max(-1, keepdims=True))
        out[:, h] = (e / e.sum(-1, keepdims=True)) @ v[:, g]
    return out


def chunk_attention(h, W, p, c):
    H, G, d = c["heads"], c["kv_heads"], c["dim"]
    T = h.shape[0]
    q = (h @ W[p + "q"].T).reshape(T, H, d)
    k = (h @ W[p + "k"].T).reshape(T, G, d)
    v = k
    rot = c.get("rot")
    if rot and rot["dims"]:
        ang, amp = yarn_angles(rot, T)
        q, k = rotate_halves(q, ang, amp, int(rot["dims"])), rotate_halves(k, ang, amp, int(rot["dims"]))
    o = softmax_attention(q, k, v, c["scale"], chunk_mask(T, int((c.get("mask") or {}).get("size", 0))))
    return o.reshape(T, H * d) @ W[p + "o"].T


def decay_recurrence(q, k, v, decay, S=None):
    """q, k [T, heads, d], v [T, heads, vd], decay [heads]: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t -> (o, S)"""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2])) if S is None else np.array(S, np.float64)
    o = np.zeros(v.shape)
    for t in range(T):
        S = np.asarray(decay, np.float64)[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def norm_then_gate(o, w, z, eps):
    return rms_norm(o, w, eps) * sigmoid(z)


def lightning(h, W, p, c, eps):
    H, d, vd = c["heads"], c["dim"], c["vdim"]
    T = h.shape[0]
    q = silu(h @ W[p + "q"].T).reshape(T, H, d)
    k = silu(h @ W[p + "k"].T).reshape(T, H, d)
    v = silu(h @ W[p + "v"].T).reshape(T, H, vd)
    o, _ = decay_recurrence(q, k, v, c["decay"])
    return norm_then_gate(o.reshape(T, H * vd), W[p + "norm"], h @ W[p + "g"].T, eps) @ W[p + "o"].T


def dense_ff(h, W, p):
    return gelu_tanh(h @ W[p + "up"].T) @ W[p + "down"].T


def route(z, top, margins=None):
    """z [T, E] biased logits -> the `top` experts with the largest ones (largest first, ties to the lower expert) and the softmax over
    those logits alone.  margins: a list that receives, per token, by how much the last chosen one beat the next"""
    ids = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    if margins is not None and top < z.shape[1]:
        s = -np.sort(-z, axis=-1)
        margins.extend((s[:, top - 1] - s[:, top]).tolist())
    c = np.take_along_axis(z, ids, axis=-1)
    e = np.exp(c - c.max(-1, keepdims=True))
    return ids, e / e.sum(-1, keepdims=True)


def expert(h, W, p):
    return relu2(h @ W[p + "up"].T) @ W[p + "down"].T


def moe_ff(h, W, p, m, margins=None):
    ids, w = route(h @ W[p + "router"].T + W[p + "router.b"], m["router"]["top"], margins)
    out = np.zeros((h.shape[0], W[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], w[t]):
            out[t] += wt * expert(h[t], W, p + "e%d." % e)
    return out + expert(h, W, p + "shared.") if m.get("shared") else out


def weight_layer(layers, i):
    while "weights_of" in layers[i]:
        i = int(layers[i]["weights_of"])
    return i


def forward(cfg, W, tokens, margins=None, operand=None):
    """-> logits [T, vocab], the sum of the copies behind every layer [n_layers, T, width]; margins: see route(); operand: what is done
    to every sublayer's normed input (a rounding: how far it alone moves the logits)"""
    tokens = np.asarray(tokens, np.int64)
    eps, s = float(cfg["norm"]["eps"]), int(cfg.get("streams", 1))
    X = np.stack([embedding(cfg, W, tokens)] * s)
    trace = []
    for i, lc in enumerate(cfg["layers"]):
        p, c, m = "l%d." % weight_layer(cfg["layers"], i), lc["mixer"], lc.get("mlp")

        def mixer(h):
            return chunk_attention(h, W, p + "mix.", c) if lc["type"] == "attention" else lightning(h, W, p + "mix.", c, eps)

        def feed_forward(h):
            return dense_ff(h, W, p + "mlp.") if m["kind"] == "dense" else moe_ff(h, W, p + "mlp.", m, margins)
        for n, f in ((1, mixer), (2, feed_forward)):
            if n == 2 and not m:
                continue
            hc = "%shc%d." % (p, n)
            h = rms_norm(stream_mixture(X, W[hc + "in"]), W[p + "norm%d" % n], eps)
            y = f(operand(h) if operand else h)
            X = stream_update(X, W[hc + "mix"], W[hc + "out"], y)
        trace.append(X.sum(0))
    z = rms_norm(X.sum(0), W["final.norm"], eps) @ W["head"].T
    cap = cfg.get("logit_softcap")
    return (cap * np.tanh(z / cap) if cap else z), np.stack(trace)


# ---------------------------------------------------------------------------------------------------------------- weights for tests
def bf16_round(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    r = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint32) << 16
    return r.view(np.float32).astype(np.float64)


def random_tosivik(rng, cfg):
    """random bf16-representable weights for a config (f64 arrays): projections ~ N(0, 1/in), norms near 1, copies that differ"""
    W = {}

    def mat(name, rows, cols, s=None):
        W[name] = bf16_round(rng.standard_normal((rows, cols)) * (s if s is not None else 1.0 / math.sqrt(cols)))

    def vec(name, n, mean=0.0, s=0.1):
        W[name] = bf16_round(mean + s * rng.standard_normal(n))

    Wd, V, s = cfg["width"], cfg["vocab"], int(cfg.get("streams", 1))
    mat("embed", V, Wd, 0.25)
    vec("final.norm", Wd, 1.0)
    mat("head", V, Wd, 2.0 / math.sqrt(Wd))
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        mat("bigram", b["buckets"] + 1, Wd, 0.5)
    for i, lc in enumerate(cfg["layers"]):
        if "weights_of" in lc:
            continue
        p, c, m = "l%d." % i, lc["mixer"], lc.get("mlp")
        q = p + "mix."
        for n in (1, 2) if m else (1,):
            vec(p + "norm%d" % n, Wd, 1.0)
            hc = "%shc%d." % (p, n)
            W[hc + "in"] = bf16_round(rng.uniform(0.2, 1.0, s) / s * 1.6)
            W[hc + "out"] = bf16_round(rng.uniform(0.3, 1.2, s))
            W[hc + "mix"] = bf16_round(0.7 * np.eye(s) + rng.uniform(-0.3, 0.5, (s, s)) / s)
        H, d, vd = c["heads"], c["dim"], c["vdim"]
        if lc["type"] == "attention":
            mat(q + "q", H * d, Wd); mat(q + "k", c["kv_heads"] * d, Wd); mat(q + "o", Wd, H * vd)
        else:
            for nm, rows in (("q", H * d), ("k", H * d), ("v", H * vd), ("g", H * vd)):
                mat(q + nm, rows, Wd)
            vec(q + "norm", H * vd, 1.0); mat(q + "o", Wd, H * vd)
        if m and m["kind"] == "dense":
            mat(p + "mlp.up", m["ff"], Wd); mat(p + "mlp.down", Wd, m["ff"])
        elif m:
            mp, E, ff = p + "mlp.", m["router"]["experts"], m["expert"]["ff"]
            for e in range(E):
                mat(mp + "e%d.up" % e, ff, Wd); mat(mp + "e%d.down" % e, Wd, ff)
            mat(mp + "router", E, Wd, 2.0 / math.sqrt(Wd)); vec(mp + "router.b", E, 0.0, 0.5)
            if m.get("shared"):
                mat(mp + "shared.up", m["shared"]["ff"], Wd); mat(mp + "shared.down", Wd, m["shared"]["ff"])
    return W
