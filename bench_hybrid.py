"""`python bench.py --hybrid`: prompt and decode throughput of the layer-list host layer (Sogodra design, or Vivazen / Kerolorn /
Sabolorn / Tosivik / Devalorn with `--hybrid-design vivazen|kerolorn|sabolorn|tosivik|devalorn`; random weights) at layer sizes of a real
model, beside the framework's closest existing model -- the 16-bit llama host layer (dense_model.cpp) -- at equal width, depth, head geometry, feed-forward size and vocabulary.  One GPU, bf16, synthetic data.  The default workload of bench.py and
its one-line contract are not touched: this option prints its own JSON line.

Per size: one prompt step of T tokens (tokens/s) and decode steps of B sequences behind `ctx` cached tokens (tokens/s), both models
driven eagerly through their step function with device-resident inputs; the hybrid model's recurrent layers have no counterpart in
the llama model, so the line also carries each model's weight bytes and the decode steps' achieved GB/s over them."""
import json
import time

import numpy as np

SIZES = {
    # name: width, heads x dim (kv heads), ff, vocab, window, delta heads x dim x vdim, gru width, layers (p = parallel, g = minGRU, d = delta)
    "1b": dict(width=2048, heads=16, kv=4, dim=128, ff=8192, vocab=32000, window=1024, dheads=16, ddim=128, dvdim=128, gru=4096, layers="pgdp"),
    "3b": dict(width=3072, heads=24, kv=8, dim=128, ff=8192, vocab=32000, window=2048, dheads=24, ddim=128, dvdim=128, gru=6144, layers="pgdp"),
    "8b": dict(width=4096, heads=32, kv=8, dim=128, ff=14336, vocab=32000, window=4096, dheads=32, ddim=128, dvdim=128, gru=8192, layers="pgdp"),
}


# Vivazen at the same widths: latent attention (heads x (dim + rot) queries over [kv_rank | rot] page rows, window) and attention behind
# a convolution (heads / kv heads as above, capped scores, mixed head weights), gelu gate/up; the fourth layer runs on the first one's weights
VIVAZEN = {
    "1b": dict(l_heads=16, l_dim=64, l_rot=64, l_rank=192, l_vdim=64, taps=4, layers="laal"),
    "3b": dict(l_heads=24, l_dim=64, l_rot=64, l_rank=192, l_vdim=64, taps=4, layers="laal"),
    "8b": dict(l_heads=32, l_dim=128, l_rot=64, l_rank=192, l_vdim=128, taps=4, layers="laal"),
}


# Kerolorn at the same widths: attention with the llama geometry (window, kept first tokens, rotation on half of the head), input
# convolution, and a mixture of experts whose ACTIVE size equals the llama feed-forward: `top` experts + the shared one, each ff / 4
KEROLORN = {
    "1b": dict(experts=16, top=3, keep=64, taps=4, layers=4),
    "3b": dict(experts=16, top=3, keep=64, taps=4, layers=4),
    "8b": dict(experts=16, top=3, keep=64, taps=4, layers=4),
}


# Sabolorn at the same widths: a state-space layer (heads x 64, state 128, inner = 2 width), attention with the llama geometry behind
# a convolution with a distance bias, latent attention with a query latent, and a second latent layer on the first one's pages; the
# state-space layer has a relu^2 feed-forward of the llama size, the others a mixture of experts whose ACTIVE size equals it (`top`
# experts of ff / 4 among 16 in 4 groups of which 2 stay open); a token side input of 256 columns per layer
SABOLORN = {
    "1b": dict(s_heads=64, s_vdim=64, s_state=128, s_groups=8, l_heads=16, l_dim=64, l_rot=64, l_rank=192, l_vdim=64, q_rank=768, taps=4,
               experts=16, top=4, groups=4, keep=2, side=256, layers="mall"),
    "3b": dict(s_heads=96, s_vdim=64, s_state=128, s_groups=8, l_heads=24, l_dim=64, l_rot=64, l_rank=192, l_vdim=64, q_rank=1024, taps=4,
               experts=16, top=4, groups=4, keep=2, side=256, layers="mall"),
    "8b": dict(s_heads=128, s_vdim=64, s_state=128, s_groups=8, l_heads=32, l_dim=128, l_rot=64, l_rank=192, l_vdim=128, q_rank=1536, taps=4,
               experts=16, top=4, groups=4, keep=2, side=256, layers="mall"),
}


# Tosivik at the same widths: linear attention with a constant decay (heads of 128 x 128) and attention with the llama geometry inside
# chunks a little larger than the others' windows (a token behind 2048 cached ones sees 949 keys at 1b, 2049 at 3b and 8b), in turn; four residual streams; the first layer has a gelu feed-forward of the
# llama size, the others relu^2 experts whose ACTIVE size equals it (`top` experts + the shared one, each ff / 4); the fourth layer runs
# on the second one's weights
TOSIVIK = {
    "1b": dict(l_heads=16, l_dim=128, l_vdim=128, streams=4, experts=16, top=3, buckets=40009, layers="lala"),
    "3b": dict(l_heads=24, l_dim=128, l_vdim=128, streams=4, experts=16, top=3, buckets=40009, layers="lala"),
    "8b": dict(l_heads=32, l_dim=128, l_vdim=128, streams=4, experts=16, top=3, buckets=40009, layers="lala"),
}


# Devalorn at the same widths: attention with the llama geometry (window, kept first tokens, a gate per head; at 3b its values are twice as
# wide) beside time mixing (width / 64 heads of 64) with a dense silu feed-forward of the llama size, and attention with a distance bias
# and a query temperature with a mixture of experts whose ACTIVE size equals it (`top` experts of ff / 4), in turn; the fourth layer
# reads the second one's keys and values
DEVALORN = {
    "1b": dict(vdim=128, rank=64, rdim=64, experts=16, top=4, keep=64, layers="paps"),
    "3b": dict(vdim=256, rank=64, rdim=64, experts=16, top=4, keep=64, layers="paps"),
    "8b": dict(vdim=128, rank=64, rdim=64, experts=16, top=4, keep=64, layers="paps"),
}


def devalorn_config(s, v):
    left = {"dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "mask": {"keep_first": v["keep"], "size": s["window"]}, "scale": s["dim"] ** -0.5,
            "rot": {"base": 500000.0, "dims": s["dim"]}, "vdim": v["vdim"]}
    par = {"left": left, "left_scale": 1.1, "right": {"dim": v["rdim"], "heads": s["width"] // v["rdim"]}, "right_scale": 0.8}
    att = {"dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "mask": {"size": s["window"] + 64}, "q_temp": {"coef": 0.1, "every": 1024},
           "scale": s["dim"] ** -0.5, "vdim": s["dim"]}
    dense = {"ff": s["ff"], "kind": "dense"}
    moe = {"expert": {"ff": s["ff"] // 4}, "kind": "moe", "router": {"experts": v["experts"], "scale": 1.5, "top": v["top"]}}
    kinds = {"p": {"type": "parallel", "mixer": par, "mlp": dense}, "a": {"type": "attention", "mixer": att, "mlp": moe},
             "s": {"type": "attention", "mixer": dict(att, kv_from=v["layers"].index("a")), "mlp": moe}}
    return {"architecture": "Devalorn", "layers": [kinds[c] for c in v["layers"]], "norm": {"eps": 1e-5}, "vocab": s["vocab"], "width": s["width"]}


def devalorn_shapes(cfg, rank=64):
    W, sh = cfg["width"], {}
    sh["embed"], sh["final.norm"], sh["head"] = (cfg["vocab"], W), (W,), (cfg["vocab"], W)

    def attention(q, c):
        sh[q + "q"], sh[q + "o"] = (c["heads"] * c["dim"], W), (W, c["heads"] * c["vdim"])
        if "kv_from" not in c:
            sh[q + "k"], sh[q + "v"] = (c["kv_heads"] * c["dim"], W), (c["kv_heads"] * c["vdim"], W)
    for i, lc in enumerate(cfg["layers"]):
        p, c, mlp = "l%d." % i, lc["mixer"], lc["mlp"]
        m = p + "mlp."
        sh[p + "norm1"], sh[p + "norm2"] = (W,), (W,)
        if lc["type"] == "parallel":
            attention(p + "mix.left.", c["left"])
            sh[p + "mix.left.g"] = (c["left"]["heads"], W)
            q, H, d = p + "mix.right.", c["right"]["heads"], c["right"]["dim"]
            for n in "rkvgw":
                sh[q + "mu." + n] = (W,)
            for n in "rkvg":
                sh[q + n] = (H * d, W)
            sh[q + "w1"], sh[q + "w2"], sh[q + "w0"], sh[q + "u"] = (rank, W), (H * d, rank), (H * d,), (H, d)
            sh[q + "norm"], sh[q + "o"] = (H * d,), (W, H * d)
        else:
            attention(p + "mix.", c)
            sh[p + "mix.q.norm"] = (c["heads"] * c["dim"],)
            if "kv_from" not in c:
                sh[p + "mix.k.norm"] = (c["kv_heads"] * c["dim"],)
        for e in ([""] if mlp["kind"] == "dense" else ["e%d." % e for e in range(mlp["router"]["experts"])]):
            ff = mlp["ff"] if mlp["kind"] == "dense" else mlp["expert"]["ff"]
            sh[m + e + "gate"], sh[m + e + "up"], sh[m + e + "down"] = (ff, W), (ff, W), (W, ff)
        if mlp["kind"] == "moe":
            sh[m + "router"] = (mlp["router"]["experts"], W)
    return sh


def tosivik_config(s, v):
    lin = {"decay": [float(np.exp(-2.0 ** (-8.0 * (i + 1) / v["l_heads"]))) for i in range(v["l_heads"])], "dim": v["l_dim"], "heads": v["l_heads"],
           "vdim": v["l_vdim"]}
    att = {"dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "mask": {"size": s["window"] + 76}, "scale": 1.1 * s["dim"] ** -0.5, "vdim": s["dim"],
           "rot": {"base": 200000.0, "dims": s["dim"], "scaling": {"factor": 8.0, "fast": 24.0, "original": 4096, "slow": 2.0}}}
    dense = {"ff": s["ff"], "kind": "dense"}
    moe = {"expert": {"ff": s["ff"] // 4}, "kind": "moe", "router": {"experts": v["experts"], "top": v["top"]}, "shared": {"ff": s["ff"] // 4}}
    layers, first = [], None
    for i, c in enumerate(v["layers"]):
        e = {"type": "lightning" if c == "l" else "attention", "mixer": lin if c == "l" else att, "mlp": dense if i == 0 else moe}
        if c == "a" and first is not None:
            e["weights_of"] = first
        first = i if c == "a" and first is None else first
        layers.append(e)
    return {"architecture": "Tosivik", "embedding": {"bigram": {"buckets": v["buckets"], "mul_cur": 31, "mul_prev": 1009}, "scale": 2.0}, "layers": layers,
            "logit_softcap": 30.0, "norm": {"eps": 1e-5}, "streams": v["streams"], "vocab": s["vocab"], "width": s["width"]}


def tosivik_shapes(cfg):
    W, sh, S = cfg["width"], {}, cfg["streams"]
    sh["embed"], sh["final.norm"], sh["head"], sh["bigram"] = (cfg["vocab"], W), (W,), (cfg["vocab"], W), (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    for i, lc in enumerate(cfg["layers"]):
        if "weights_of" in lc:
            continue
        p, c, mlp = "l%d." % i, lc["mixer"], lc["mlp"]
        q, m = p + "mix.", p + "mlp."
        for n in (1, 2):
            sh[p + "norm%d" % n] = (W,)
            sh[p + "hc%d.in" % n], sh[p + "hc%d.out" % n], sh[p + "hc%d.mix" % n] = (S,), (S,), (S, S)
        H, d, vd = c["heads"], c["dim"], c["vdim"]
        sh[q + "q"], sh[q + "o"] = (H * d, W), (W, H * vd)
        if lc["type"] == "attention":
            sh[q + "k"] = (c["kv_heads"] * d, W)
        else:
            sh[q + "k"], sh[q + "v"], sh[q + "g"], sh[q + "norm"] = (H * d, W), (H * vd, W), (H * vd, W), (H * vd,)
        if mlp["kind"] == "dense":
            sh[m + "up"], sh[m + "down"] = (mlp["ff"], W), (W, mlp["ff"])
        else:
            for e in ["e%d" % e for e in range(mlp["router"]["experts"])] + ["shared"]:
                ff = mlp["shared" if e == "shared" else "expert"]["ff"]
                sh[m + e + ".up"], sh[m + e + ".down"] = (ff, W), (W, ff)
            sh[m + "router"], sh[m + "router.b"] = (mlp["router"]["experts"], W), (mlp["router"]["experts"],)
    return sh


def sabolorn_config(s, v):
    ssm = {"conv": v["taps"], "groups": v["s_groups"], "heads": v["s_heads"], "norm_groups": v["s_groups"], "state": v["s_state"], "vdim": v["s_vdim"]}
    att = {"conv": v["taps"], "dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "scale": s["dim"] ** -0.5, "vdim": s["dim"]}
    lat = {"dim": v["l_dim"], "heads": v["l_heads"], "kv_rank": v["l_rank"], "q_rank": v["q_rank"], "rot_dim": v["l_rot"], "vdim": v["l_vdim"],
           "scale": (v["l_dim"] + v["l_rot"]) ** -0.5,
           "rot": {"base": 10000.0, "dims": v["l_rot"], "scaling": {"factor": 8.0, "fast": 24.0, "original": 4096, "slow": 2.0}}}
    moe = {"expert": {"ff": s["ff"] // 4}, "kind": "moe",
           "router": {"experts": v["experts"], "groups": {"count": v["groups"], "keep": v["keep"]}, "top": v["top"]}}
    dense = {"ff": s["ff"], "kind": "dense"}
    layers, first = [], None
    for i, c in enumerate(v["layers"]):
        if c == "m":
            layers.append({"type": "mamba2", "mixer": ssm, "mlp": dense})
        elif c == "a":
            layers.append({"type": "attention", "mixer": att, "mlp": moe})
        else:
            layers.append({"type": "latent_attention", "mixer": lat if first is None else dict(lat, kv_from=first), "mlp": moe})
            first = i if first is None else first
    return {"architecture": "Sabolorn", "embedding": {"scale": 0.5}, "layers": layers, "logit_softcap": 30.0, "norm": {"eps": 1e-5},
            "token_side": {"dim": v["side"]}, "vocab": s["vocab"], "width": s["width"]}


def sabolorn_shapes(cfg):
    W, sh, n = cfg["width"], {}, len(cfg["layers"])
    sh["embed"], sh["final.norm"], sh["side.embed"] = (cfg["vocab"], W), (W,), (cfg["vocab"], n * cfg["token_side"]["dim"])
    for i, lc in enumerate(cfg["layers"]):
        p, c, mlp = "l%d." % i, lc["mixer"], lc["mlp"]
        q, m = p + "mix.", p + "mlp."
        sh[p + "norm1"], sh[p + "dwa"] = (W,), (i + 2,)
        sh[p + "side.gate"], sh[p + "side.proj"], sh[p + "side.norm"] = (cfg["token_side"]["dim"], W), (W, cfg["token_side"]["dim"]), (W,)
        if lc["type"] == "mamba2":
            inner, gn = c["heads"] * c["vdim"], c["groups"] * c["state"]
            sh[q + "in"], sh[q + "conv"], sh[q + "conv.b"] = (2 * inner + 2 * gn + c["heads"], W), (inner + 2 * gn, c["conv"]), (inner + 2 * gn,)
            sh[q + "dt_bias"], sh[q + "A_log"], sh[q + "D"], sh[q + "norm"], sh[q + "o"] = (c["heads"],), (c["heads"],), (c["heads"],), (inner,), (W, inner)
        elif lc["type"] == "attention":
            H, G, d, vd, t = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"]
            for nme, rows in (("q", H * d), ("k", G * d), ("v", G * vd)):
                sh[q + nme], sh[q + nme + ".b"], sh[q + nme + ".conv"] = (rows, W), (rows,), (rows, t)
            sh[q + "r1"], sh[q + "r2"], sh[q + "o"] = (H,), (H,), (W, H * vd)
        else:
            H, d, r, vd, rank, qr = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"], c["q_rank"]
            sh[q + "dq"], sh[q + "dq.norm"], sh[q + "uq"] = (qr, W), (qr,), (H * (d + r), qr)
            if "kv_from" not in c:
                sh[q + "dkv"], sh[q + "dkv.norm"] = (rank + r, W), (rank,)
            sh[q + "uk"], sh[q + "uv"], sh[q + "g"], sh[q + "o"] = (H * d, rank), (H * vd, rank), (H * vd, W), (W, H * vd)
        if mlp and mlp["kind"] == "dense":
            sh[m + "up"], sh[m + "down"] = (mlp["ff"], W), (W, mlp["ff"])
        elif mlp:
            ff, E = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(E):
                sh[m + "e%d.gate" % e], sh[m + "e%d.up" % e], sh[m + "e%d.down" % e] = (ff, W), (ff, W), (W, ff)
            sh[m + "router"], sh[m + "correction"] = (E, W), (E,)
    return sh


def kerolorn_config(s, v):
    att = {"dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "vdim": s["dim"], "scale": 1.2 * s["dim"] ** -0.5,
           "mask": {"size": s["window"], "keep_first": v["keep"]},
           "rot": {"base": 500000.0, "dims": s["dim"] // 2, "scaling": {"factor": 4.0, "fast": 24.0, "original": 4096, "slow": 2.0}}}
    mlp = {"expert": {"ff": s["ff"] // 4}, "kind": "moe", "router": {"experts": v["experts"], "scale": 2.0, "top": v["top"]},
           "shared": {"ff": s["ff"] // 4}}
    return {"architecture": "Kerolorn", "canon": {"taps": v["taps"]}, "layers": [{"type": "attention", "mixer": att, "mlp": mlp}] * v["layers"],
            "logit_scale": 1.5, "norm": {"eps": 1e-6}, "vocab": s["vocab"], "width": s["width"]}


def kerolorn_shapes(cfg):
    W, sh = cfg["width"], {}
    sh["embed"], sh["final.norm"], sh["head"] = (cfg["vocab"], W), (W,), (cfg["vocab"], W)
    for i, lc in enumerate(cfg["layers"]):
        p, c, mlp = "l%d." % i, lc["mixer"], lc["mlp"]
        q, m = p + "mix.", p + "mlp."
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            sh[p + n] = (W,)
        sh[p + "canon1"] = (W, cfg["canon"]["taps"])
        H, G, d, vd = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
        sh[q + "q"], sh[q + "k"], sh[q + "v"], sh[q + "temp"], sh[q + "o"] = (H * d, W), (G * d, W), (G * vd, W), (H,), (W, H * vd)
        ff, E, fs = mlp["expert"]["ff"], mlp["router"]["experts"], mlp["shared"]["ff"]
        for e in range(E):
            sh[m + "e%d.gate" % e], sh[m + "e%d.up" % e], sh[m + "e%d.down" % e] = (ff, W), (ff, W), (W, ff)
        sh[m + "router"], sh[m + "correction"] = (E, W), (E,)
        sh[m + "shared.gate"], sh[m + "shared.up"], sh[m + "shared.down"], sh[m + "shared.sg"] = (fs, W), (fs, W), (W, fs), (1, W)
    return sh


def vivazen_config(s, v):
    lat = {"dim": v["l_dim"], "heads": v["l_heads"], "kv_rank": v["l_rank"], "rot_dim": v["l_rot"], "vdim": v["l_vdim"],
           "scale": (v["l_dim"] + v["l_rot"]) ** -0.5, "mask": {"size": s["window"]},
           "rot": {"base": 10000.0, "dims": v["l_rot"], "scaling": {"factor": 8.0, "fast": 24.0, "original": 4096, "slow": 2.0}}}
    att = {"conv": v["taps"], "dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "scale": s["dim"] ** -0.5, "softcap": 30.0, "vdim": s["dim"]}
    mlp = {"ff": s["ff"], "kind": "dense"}
    layers, first = [], {}
    for i, c in enumerate(v["layers"]):
        e = {"type": "latent_attention" if c == "l" else "attention", "mixer": lat if c == "l" else att, "mlp": mlp}
        if c == "l" and "l" in first:
            e["weights_of"] = first["l"]
        first.setdefault(c, i)
        layers.append(e)
    return {"architecture": "Vivazen", "layers": layers, "norm": {"eps": 1e-6, "groups": 8}, "postln_alpha": 2.0, "vocab": s["vocab"], "width": s["width"]}


def vivazen_shapes(cfg):
    W, sh = cfg["width"], {}
    sh["embed"], sh["final.norm"], sh["head"] = (cfg["vocab"], W), (W,), (cfg["vocab"], W)
    for i, lc in enumerate(cfg["layers"]):
        if "weights_of" in lc:
            continue
        p, c = "l%d." % i, lc["mixer"]
        q = p + "mix."
        sh[p + "norm1"] = (W,)
        if lc["type"] == "latent_attention":
            H, d, r, vd, rank = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
            sh[q + "q"], sh[q + "dkv"], sh[q + "dkv.norm"], sh[q + "uk"], sh[q + "uv"] = (H * (d + r), W), (rank + r, W), (rank,), (H * d, rank), (H * vd, rank)
            sh[q + "sink"], sh[q + "g"], sh[q + "o"] = (H,), (H, W), (W, H * vd)
        else:
            H, G, d, vd, t = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * vd)):
                sh[q + n], sh[q + n + ".conv"] = (rows, W), (rows, t)
            sh[q + "q.norm"], sh[q + "k.norm"], sh[q + "talk"], sh[q + "o"] = (H * d,), (G * d,), (H, H), (W, H * vd)
        if lc.get("mlp"):
            ff = lc["mlp"]["ff"]
            sh[p + "norm2"], sh[p + "mlp.gate"], sh[p + "mlp.up"], sh[p + "mlp.down"] = (W,), (ff, W), (ff, W), (W, ff)
    return sh


def sogodra_config(s):
    att = {"dim": s["dim"], "heads": s["heads"], "kv_heads": s["kv"], "vdim": s["dim"], "scale": s["dim"] ** -0.5, "mask": {"size": s["window"]},
           "rot": {"base": 500000.0, "dims": s["dim"], "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    right = {"conv": 4, "dim": s["ddim"], "heads": s["dheads"], "kv_heads": s["dheads"], "vdim": s["dvdim"]}
    mlp = {"ff": s["ff"], "kind": "dense", "limit": 7.0}
    kinds = {"p": lambda: {"type": "parallel", "mixer": {"left": att, "right": right, "left_scale": 1.0, "right_scale": 1.0}, "mlp": mlp},
             "g": lambda: {"type": "mingru", "mixer": {"width": s["gru"]}, "mlp": mlp},
             "d": lambda: {"type": "delta", "mixer": right, "mlp": mlp}}
    return {"architecture": "Sogodra", "layers": [kinds[c]() for c in s["layers"]], "norm": {"eps": 1e-5}, "vocab": s["vocab"], "width": s["width"]}


def sogodra_shapes(cfg, a_rank=64, g_rank=64):
    """tensor name -> shape for a config (the low-rank parts' ranks are free: the design reads them from the tensors)"""
    W, sh = cfg["width"], {}
    sh["embed"], sh["final.norm"], sh["head"] = (cfg["vocab"], W), (W,), (cfg["vocab"], W)

    def delta(p, c, lr):
        H, G, d, vd, t = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"]
        for n, r in (("q", G * d), ("k", G * d), ("v", H * vd)):
            sh[p + n], sh[p + n + ".conv"] = (r, W), (r, t)
        sh[p + "b"], sh[p + "A_log"], sh[p + "norm"], sh[p + "o"] = (H, W), (H,), (vd,), (W, H * vd)
        if lr:
            sh[p + "a1"], sh[p + "a2"], sh[p + "dt_bias"], sh[p + "g1"], sh[p + "g2"] = (a_rank, W), (H * d, a_rank), (H * d,), (g_rank, W), (H * vd, g_rank)
        else:
            sh[p + "a"], sh[p + "dt_bias"], sh[p + "g"] = (H, W), (H,), (H * vd, W)
    for i, lc in enumerate(cfg["layers"]):
        p, m = "l%d." % i, lc["mixer"]
        sh[p + "norm1"] = (W,)
        if lc["type"] == "parallel":
            c, q = m["left"], p + "mix.left."
            sh[q + "q"], sh[q + "k"], sh[q + "v"] = (c["heads"] * c["dim"], W), (c["kv_heads"] * c["dim"], W), (c["kv_heads"] * c["vdim"], W)
            sh[q + "q.norm"], sh[q + "k.norm"], sh[q + "sink"], sh[q + "o"] = (c["dim"],), (c["dim"],), (c["heads"],), (W, c["heads"] * c["vdim"])
            delta(p + "mix.right.", m["right"], True)
        elif lc["type"] == "delta":
            delta(p + "mix.", m, False)
        else:
            w = m["width"]
            for n in ("z", "x", "g"):
                sh[p + "mix." + n] = (w, W)
            sh[p + "mix.z.b"], sh[p + "mix.x.b"], sh[p + "mix.o"] = (w,), (w,), (W, w)
        if lc.get("mlp"):
            ff = lc["mlp"]["ff"]
            sh[p + "norm2"], sh[p + "mlp.gate"], sh[p + "mlp.up"], sh[p + "mlp.down"] = (W,), (ff, W), (ff, W), (W, ff)
    return sh


def build_hybrid(cfg, max_tokens, slots):
    """random weights generated on the GPU, concatenated as the loader does it, handed over as device bf16"""
    import torch
    from candle_vllm_amd import hybrid_model as hm
    shapes = {"Vivazen": vivazen_shapes, "Kerolorn": kerolorn_shapes, "Sogodra": sogodra_shapes, "Sabolorn": sabolorn_shapes,
              "Tosivik": tosivik_shapes, "Devalorn": devalorn_shapes}[cfg["architecture"]](cfg)
    spec = hm.SPECS[cfg["architecture"]](cfg, shapes)
    m = hm.HybridModel(spec, dtype="bfloat16", block_size=64, state_slots=slots)
    g = torch.Generator(device="cuda").manual_seed(7)
    nbytes = 0

    def rnd(shape, name):
        fan = shape[-1] if len(shape) > 1 else 1
        if name.split(".")[-1].startswith("norm") or name.endswith(".temp"):
            return (1 + 0.02 * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name.endswith(".correction"):
            return (0.05 * torch.rand(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name.endswith(".router"):
            return (2.0 * fan ** -0.5 * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name == "embed":
            return ((0.25 if cfg["architecture"] == "Sabolorn" else 1.0) * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name.endswith(".r1") or name.endswith(".r2"):                  # the distance bias: positive rates
            return (0.1 + torch.rand(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if ".mu." in name:                                                # how much of the token before a mixture takes
            return torch.rand(shape, generator=g, device="cuda").to(torch.bfloat16)
        if name.endswith(".w0"):                                          # decays between about 0.7 and 0.998 per token
            return (-6 + 5 * torch.rand(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name.endswith(".dwa"):
            return torch.full(shape, 1.0 / shape[0], device="cuda").to(torch.bfloat16)
        if ".hc" in name:                                                 # mixing of the residual streams: near the identity, every stream takes part
            n = shape[0]
            base = 0.8 * torch.eye(n, device="cuda") + 0.2 / n if name.endswith(".mix") else torch.full(shape, 1.0 / n if name.endswith(".in") else 0.7, device="cuda")
            return (base + 0.05 * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)
        if name.endswith(".talk"):
            return (torch.eye(shape[0], device="cuda") + 0.1 * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)
        s = 0.5 if name.endswith(".conv") else 0.3 if name.endswith("canon1") else (fan ** -0.5 if len(shape) > 1 else 0.3)
        return (s * torch.randn(shape, generator=g, device="cuda")).to(torch.bfloat16)

    def put(layer, which, names, axis=0):
        nonlocal nbytes
        if isinstance(names[0], hm.Constants):
            v = np.ascontiguousarray(names[0].values)
            hm._check(hm.lib.mi355_hybrid_set_weight_f32(m.h, layer, which, v.ctypes.data, v.size), "set_weight_f32")
            return
        names = [n.name if isinstance(n, hm.HeadTranspose) else n for n in names]       # random values: the transposed layout is as random
        ts = [None if not n else torch.zeros((n.rows, n.cols), dtype=torch.bfloat16, device="cuda") if isinstance(n, hm.ZeroRows) else rnd(shapes[n], n)
              for n in names]
        if which == hm.HW_IN_BIAS:
            rows = [shapes[p][0] for p in spec.slots[layer][hm.HW_IN_PROJ]]
            ts = [t if t is not None else torch.zeros(r, dtype=torch.bfloat16, device="cuda") for t, r in zip(ts, rows)]
        t = torch.cat([x if axis else x.reshape(-1) for x in ts], dim=1 if axis else 0).contiguous()
        nbytes += t.numel() * 2
        hm._check(hm.lib.mi355_hybrid_set_weight_dev(m.h, layer, which, t.data_ptr(), t.numel(), torch.cuda.current_stream().cuda_stream), "set_weight_dev")
        torch.cuda.synchronize()
    globals_ = spec.globals_() if hasattr(spec, "globals_") else {hm.HW_EMBED: "embed", hm.HW_FINAL_NORM: "final.norm", hm.HW_HEAD: "head"}
    for which, name in globals_.items():
        put(-1, which, [name])
    for i, slots_ in enumerate(spec.slots):
        for which, names in slots_.items():
            put(i, which, names, axis=1 if (which == hm.HW_OUT_PROJ and len(names) > 1) else 0)
    m.alloc_cache(-(-max_tokens // 64))
    return m, nbytes


def time_calls(call, sync, reps=5, settle_ms=200.0):
    t, n = 0.0, 0
    while t < settle_ms and n < 20:
        t0 = time.perf_counter(); call(); sync(); t += (time.perf_counter() - t0) * 1e3; n += 1
    d = []
    for _ in range(reps):
        sync(); t0 = time.perf_counter(); call(); sync(); d.append(time.perf_counter() - t0)
    return sorted(d)[len(d) // 2]


def run_size(name, T=2048, B=8, ctx=2048, dec_steps=16, design="sogodra"):
    import torch
    from candle_vllm_amd import dense_model as DM
    from candle_vllm_amd.block_engine import BlockEngine
    from candle_vllm_amd.step_engine import StepEngine
    from oracle.dense_llama import DenseConfig
    s = SIZES[name]
    extra = {"vivazen": VIVAZEN, "kerolorn": KEROLORN, "sabolorn": SABOLORN, "tosivik": TOSIVIK, "devalorn": DEVALORN}.get(design, {}).get(name, {})
    cfg = (vivazen_config(s, extra) if design == "vivazen" else kerolorn_config(s, extra) if design == "kerolorn" else
           sabolorn_config(s, extra) if design == "sabolorn" else tosivik_config(s, extra) if design == "tosivik" else devalorn_config(s, extra) if design == "devalorn" else
           sogodra_config(s))
    rng = np.random.default_rng(5)
    out = {"size": name, "design": design, "shape": dict(s, **extra), "prompt_tokens": T, "decode_batch": B,
           "decode_ctx": ctx}
    sync = torch.cuda.synchronize
    # ---- hybrid: prompt step, then B sequences decoding behind ctx tokens
    hyb, wbytes = build_hybrid(cfg, max(T, B * (ctx + 1024)) + 64, slots=max(4, B))
    eng = StepEngine(hyb, max(T, B * (ctx + 1024)) + 64)
    toks = rng.integers(0, s["vocab"], T).tolist()

    def prompt_h():
        eng.feed("p", toks)
        eng.step(["p"])
        eng.finish("p")
    dt = time_calls(prompt_h, sync, reps=3)
    out["hybrid_prompt_tok_s"] = round(T / dt, 1)
    ids = ["s%d" % i for i in range(B)]
    for r in ids:
        eng.feed(r, rng.integers(0, s["vocab"], ctx).tolist())
        eng.step([r])

    def decode_h():
        for _ in range(dec_steps):
            for r in ids:
                eng.feed(r, [int(rng.integers(0, s["vocab"]))])          # (a mixture of experts routes by token: no two sequences the same one)
            eng.step(ids)
    dt = time_calls(decode_h, sync, reps=3)
    out["hybrid_decode_tok_s"] = round(B * dec_steps / dt, 1)
    out["hybrid_decode_ms_per_step"] = round(dt / dec_steps * 1e3, 3)
    out["hybrid_weight_GB"] = round(wbytes / 1e9, 3)
    out["hybrid_decode_weight_GBs"] = round(wbytes * dec_steps / dt / 1e9, 1)
    del eng, hyb
    torch.cuda.empty_cache()
    # ---- the llama host layer at equal size
    n_layers = len(cfg["layers"])
    dc = DenseConfig(hidden=s["width"], n_layers=n_layers, n_heads=s["heads"], n_kv_heads=s["kv"], head_dim=s["dim"], intermediate=s["ff"],
                     vocab=s["vocab"], max_seq=8192, block_size=64)
    nblk = B * (-(-(ctx + 64) // 64)) + (-(-T // 64)) + 2
    gm = DM.DenseLlama(dc, max_batch=B, max_blocks_per_seq=-(-max(T, ctx + 64) // 64) + 1, kv_layout=DM.KV_PAGED)
    gm.load_synthetic()
    gm.alloc_kv_cache(nblk)
    be = BlockEngine(64, nblk, 0)
    seq = be.new_sequence(1000, toks)
    be.allocate([seq], chunk=T)
    meta = be.prepare_prompt([seq])
    dt = time_calls(lambda: gm.forward(meta, is_prefill=True, sync=False), sync, reps=3)
    out["llama_prompt_tok_s"] = round(T / dt, 1)
    be.free_sequence(seq)
    seqs = []
    for i in range(B):
        q = be.new_sequence(i, rng.integers(0, s["vocab"], ctx + 1).tolist())
        be.allocate([q], chunk=ctx + 64)
        seqs.append(q)
    dmeta = be.prepare_decode(seqs)

    def decode_l():
        for _ in range(dec_steps):
            gm.forward(dmeta, is_prefill=False, sync=False)
    dt = time_calls(decode_l, sync, reps=3)
    out["llama_decode_tok_s"] = round(B * dec_steps / dt, 1)
    out["llama_decode_ms_per_step"] = round(dt / dec_steps * 1e3, 3)
    out["llama_weight_GB"] = round(gm.weight_bytes() / 1e9, 3)
    out["llama_decode_weight_GBs"] = round(gm.weight_bytes() * dec_steps / dt / 1e9, 1)
    out["prompt_ratio_hybrid_over_llama"] = round(out["hybrid_prompt_tok_s"] / out["llama_prompt_tok_s"], 3)
    out["decode_ratio_hybrid_over_llama"] = round(out["hybrid_decode_tok_s"] / out["llama_decode_tok_s"], 3)
    del gm
    torch.cuda.empty_cache()
    return out


def main(sizes="1b,3b", prompt_tokens=2048, batch=8, ctx=2048, design="sogodra"):
    if design not in ("sogodra", "vivazen", "kerolorn", "sabolorn", "tosivik", "devalorn"):
        raise SystemExit("--hybrid-design: sogodra, vivazen, kerolorn, sabolorn, tosivik or devalorn")
    res = [run_size(n.strip(), T=prompt_tokens, B=batch, ctx=ctx, design=design) for n in sizes.split(",") if n.strip()]
    print(json.dumps({"metric": "hybrid_vs_llama_throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
                      "note": "%s layer-list host layer beside the 16-bit llama host layer at equal sizes; the hybrid side's decode steps replay "
                              "a hipGraph, the rest runs eagerly" % design.capitalize(), "sizes": res}))
