"""Small random Nerenex, Safolorn, Segetar and Fororax models for the tests: configuration, weights (bfloat16-representable), checkpoint directories."""
import json
import os
import struct

import numpy as np


def bf16(a):
    """Round to bfloat16 and back (nearest even)."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return (((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32)).view(np.float32)


def attention(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, base=10000.0, scale=None, ff=None):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim}, "scale": scale or (dim + rot_dim) ** -0.5}}


def recurrent(width, blocks, conv, ff=None):
    return {"type": "rglru", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def config(width, vocab, layers, eps=1e-5, mult=0.8, buckets=97, mul_prev=31, mul_cur=5):
    return {"architecture": "Nerenex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}


def sink_attention(heads, dim, rot_dim, vdim, kv_rank, base=10000.0, yarn=None, scale=None, kv_from=None, mlp=None):
    """yarn: (factor, original, fast, slow)"""
    rot = {"base": base, "dims": rot_dim}
    if yarn:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": rot, "scale": scale or (dim + rot_dim) ** -0.5}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mlp": mlp, "mixer": mixer}


def glu(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def experts(n, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}


def safolorn(width, vocab, side, layers, eps=1e-5):
    return {"architecture": "Safolorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "token_side": {"dim": side}, "layers": layers}


NERENEX = {
    # nothing is a multiple of 32; value size, query size and ranks all differ; attention without, recurrence with a feed-forward
    "odd": config(100, 131, [attention(3, 20, 6, 36, 44, 52, 21, base=500.0), recurrent(66, 3, 3, ff=75), attention(5, 9, 10, 12, 31, 70, 50, ff=41)],
                  eps=1e-3, mult=0.45),
    # several heads tiles, a rank of more than one padded size, one recurrent block, a long window
    "wide": config(288, 260, [recurrent(256, 1, 2, ff=416), attention(20, 64, 32, 48, 192, 256, 130, ff=416), recurrent(192, 6, 5)], mult=0.6),
    # the largest compile-time extents of the attention kernels
    "deep": config(320, 203, [attention(16, 128, 64, 128, 160, 512, 90, base=1e6), attention(7, 96, 40, 120, 72, 300, 33, ff=130)], eps=1e-6, mult=0.9),
    "tiny": config(40, 61, [recurrent(24, 2, 1, ff=33), attention(2, 8, 4, 8, 16, 24, 7, ff=50), attention(1, 12, 2, 20, 8, 9, 1)], buckets=11),
}
SHORT, LONG = (3.0, 40, 6.0, 1.0), (2.5, 96, 9.0, 0.5)
SAFOLORN = {
    # nothing is a multiple of 32; two caches, each read by a later layer; a layer without feed-forward; all experts chosen
    "sinks": safolorn(100, 131, 10, [sink_attention(3, 20, 6, 36, 52, 500.0, SHORT, mlp=glu(75, 0.7)), sink_attention(5, 9, 10, 12, 70, mlp=experts(7, 3, 41)),
                                     sink_attention(4, 12, 6, 20, 52, 500.0, SHORT, kv_from=0), sink_attention(2, 9, 10, 8, 70, kv_from=1, mlp=experts(5, 5, 33))],
                      eps=1e-3),
    # more heads than a row tile, ranks and heads of several padded sizes, one cache read by layers of other head counts
    "shared": safolorn(288, 260, 40, [sink_attention(20, 64, 32, 48, 256, 1e5, LONG, mlp=glu(416, 1.5)), sink_attention(17, 40, 32, 64, 256, 1e5, LONG, kv_from=0, mlp=experts(20, 2, 72)),
                                      sink_attention(3, 128, 64, 128, 512, 1e6, SHORT, mlp=experts(12, 1, 160)), sink_attention(6, 32, 32, 96, 256, 1e5, LONG, kv_from=0, mlp=glu(130, 0.3))]),
    "one": safolorn(40, 61, 1, [sink_attention(1, 5, 2, 3, 7, mlp=experts(1, 1, 9)), sink_attention(2, 8, 4, 8, 24, yarn=(1.0, 64, 4.0, 2.0), mlp=glu(1, 2.0))], eps=0.1),
}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def grouped_experts(n, top, ff, groups=1, keep=1, scale=1.0):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}}


def gated_pair(heads, kv_heads, dim, vdim, window, lin_heads, lin_dim, lin_vdim, tau=16.0, rot=None, base=1e4, left=1.0, right=1.0, scale=None, mlp=None):
    """Windowed attention beside gated linear attention."""
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "scale": scale or dim ** -0.5,
                 "rot": {"base": base, "dims": dim // 2 * 2 if rot is None else rot}},
        "right": {"heads": lin_heads, "dim": lin_dim, "vdim": lin_vdim, "tau": tau}, "left_scale": left, "right_scale": right}}


def retention_pair(heads, kv_heads, dim, vdim, window, decay, lin_dim, lin_vdim, rot=None, base=1e4, scale=None, mlp=None):
    """Windowed attention beside retention, one head per entry of `decay`."""
    return {"type": "parallel_2", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "scale": scale or dim ** -0.5},
        "right": {"heads": len(decay), "dim": lin_dim, "vdim": lin_vdim, "decay": list(decay),
                  "rot": {"base": base, "dims": lin_dim // 2 * 2 if rot is None else rot}}}}


def scan(inner, state, dt_rank, conv, mlp=None):
    return {"type": "mamba1", "mlp": mlp, "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}}


def segetar(width, vocab, layers, loop=None, eps=1e-5):
    """loop: (start, stop, times)"""
    c = {"architecture": "Segetar", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


SEGETAR = {
    # nothing is a multiple of 32; a loop in the middle whose passes keep caches and states of their own; a layer without feed-forward
    "loop": segetar(100, 131, [retention_pair(6, 2, 20, 28, 21, (0.5, 0.97, 0.999), 18, 44, 12, 300.0, mlp=grouped_experts(12, 3, 41, 3, 2, 1.7)),
                               scan(75, 9, 5, 3, mlp=dense(50)), gated_pair(4, 4, 24, 10, 50, 5, 12, 20, 4.0, 10, 500.0, 0.7, -1.3),
                               scan(44, 3, 40, 2, mlp=grouped_experts(7, 2, 33))], (1, 3, 3), 1e-3),
    # several row tiles of heads, heads of several padded sizes, the loop over everything, decays from almost 1 to almost 0
    "all": segetar(288, 260, [gated_pair(24, 1, 64, 64, 130, 8, 64, 128, 1.0, left=0.5, right=2.0, mlp=dense(416)),
                              retention_pair(8, 4, 128, 96, 33, (0.99, 0.9, 0.3, 0.9995, 0.95), 96, 64, mlp=grouped_experts(24, 4, 72, 4, 1, 0.8)),
                              scan(512, 16, 20, 4, mlp=grouped_experts(16, 2, 40, 2, 2, 2.5))], (0, 3, 2), 1e-6),
    # a width that no vector load divides
    "narrow": segetar(45, 53, [scan(30, 5, 3, 3, mlp=grouped_experts(6, 2, 21, 2, 1)), retention_pair(5, 5, 7, 9, 11, (0.6, 0.98, 0.9), 10, 13, mlp=dense(37)),
                                  gated_pair(6, 3, 10, 6, 19, 2, 20, 50, 2.0, 6, mlp=grouped_experts(9, 4, 15, 3, 2, 0.6))], (1, 2, 4), 1e-4),
    "bare": segetar(40, 61, [scan(24, 2, 1, 1), gated_pair(1, 1, 5, 3, 1, 1, 3, 2, mlp=dense(1)),
                             retention_pair(2, 1, 8, 8, 7, (0.8,), 6, 5, 2, mlp=grouped_experts(2, 1, 9, 2, 1))], None, 0.1),
    "once": segetar(64, 77, [gated_pair(2, 2, 16, 16, 9, 2, 16, 16, mlp=grouped_experts(8, 2, 32, 2, 1)), scan(64, 8, 4, 4, mlp=dense(96))], (0, 1, 1)),
}


def identity_experts(n, identity, top, ff, shared, limit=1.2, shared_limit=0.8):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": n, "identity": identity, "top": top}, "shared": {"ff": shared, "limit": shared_limit}}


def far_attention(heads, kv_heads, dim, vdim, scale=None, kv_from=None, mlp=None):
    """Scores that fall with the logarithm of the distance."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mlp": mlp, "mixer": m}


def talk_attention(heads, kv_heads, dim, vdim, scale=None, mlp=None):
    """Sinks, heads mixed between softmax and values, value gates, biases."""
    return {"type": "attention_2", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}}


def fororax(width, vocab, layers, eps=1e-5, alpha=1.8, scale=1.0, cap=20.0, positions=600):
    return {"architecture": "Fororax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "postln_alpha": alpha, "embedding": {"scale": scale},
            "logit_softcap": cap, "max_positions": positions, "layers": layers}


FORORAX = {
    # nothing is a multiple of 32; a layer that reads the first one's keys with more heads of its own; a layer without feed-forward
    "far": fororax(100, 131, [far_attention(4, 2, 20, 28, mlp=identity_experts(7, 3, 2, 41, 50)), talk_attention(6, 2, 24, 10, mlp=identity_experts(5, 1, 3, 33, 20, 0.5, 2.0)),
                              far_attention(6, 2, 20, 28, kv_from=0), talk_attention(5, 5, 12, 36, mlp=identity_experts(6, 2, 1, 24, 70))], 1e-3, 1.6, 0.7, 6.0),
    # heads in one and two row tiles, key / value heads shared by a wave's heads or not, heads of several padded sizes
    "talks": fororax(288, 260, [talk_attention(24, 8, 64, 40, mlp=identity_experts(20, 4, 3, 72, 130)), talk_attention(16, 4, 128, 128, mlp=identity_experts(12, 6, 4, 160, 64)),
                                far_attention(8, 1, 96, 64, mlp=identity_experts(6, 6, 2, 40, 96)), talk_attention(32, 4, 32, 32), far_attention(5, 1, 96, 64, kv_from=2)],
                     1e-6, 2.0, 1.5, 30.0),
    # a width that no vector load divides
    "uneven": fororax(45, 53, [talk_attention(3, 1, 7, 9, mlp=identity_experts(4, 2, 2, 21, 15)), far_attention(3, 3, 10, 6, mlp=identity_experts(3, 1, 2, 37, 9))], 1e-4, 1.3, 2.0, 12.0),
    "lone": fororax(40, 61, [talk_attention(1, 1, 5, 3, mlp=identity_experts(2, 1, 1, 9, 1)), far_attention(2, 1, 8, 8, mlp=identity_experts(1, 0, 1, 12, 33))], 0.1, 1.0),
}
CONFIGS = {**NERENEX, **SAFOLORN, **SEGETAR, **FORORAX}
CLASSES = 4
# draws in which no token's choice of experts is close
SEEDS = {"narrow": 13, "loop": 23, "all": 17, "bare": 11, "once": 11, "far": 20, "talks": 20, "uneven": 20, "lone": 14}


def weights(cfg, seed, **kw):
    return {"Nerenex": nerenex_weights, "Safolorn": safolorn_weights, "Segetar": segetar_weights, "Fororax": fororax_weights}[cfg["architecture"]](cfg, seed, **kw)


def safolorn_weights(cfg, seed, clear_routes=True):
    """clear_routes: the first CLASSES coordinates of the stream hold the token's class and nothing else, and the router mostly reads
    them, with an order of the experts per class and wide gaps: no rounding changes a choice, and every expert is chosen by some class
    (experts permitting)."""
    rng = np.random.default_rng(seed)
    D, V, S, n = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"], len(cfg["layers"])
    w = {}

    def mat(name, *shape, std=None):
        w[name] = bf16(rng.standard_normal(shape) * (std or shape[-1] ** -0.5))

    def num(name):
        w[name] = bf16(rng.uniform(0.6, 1.5, ())).reshape(())

    mat("embed", V, D, std=1.0)
    mat("side.embed", V, n * S, std=1.0)
    mat("head", V, D)
    num("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x, H = p + "mix.", m["heads"]
        num(p + "norm1")
        mat(x + "q", H * (m["dim"] + m["rot_dim"]), D, std=1.6 * D ** -0.5)
        if "kv_from" not in m:
            mat(x + "dkv", m["kv_rank"] + m["rot_dim"], D)
            w[x + "dkv.norm"] = bf16(1.0 + 0.2 * rng.standard_normal(m["kv_rank"]))
        mat(x + "uk", H * m["dim"], m["kv_rank"], std=1.6 * m["kv_rank"] ** -0.5)
        mat(x + "uv", H * m["vdim"], m["kv_rank"])
        w[x + "sink"] = bf16(2.0 + 1.5 * rng.standard_normal(H))
        mat(x + "o", D, H * m["vdim"], std=2.0 * (H * m["vdim"]) ** -0.5)
        outs = [x + "o", p + "side.proj"]
        if ff:
            num(p + "norm2")
        if ff and ff["kind"] == "dense":
            mat(p + "mlp.gate", ff["ff"], D, std=1.5 * D ** -0.5)
            mat(p + "mlp.up", ff["ff"], D)
            mat(p + "mlp.down", D, ff["ff"])
            outs.append(p + "mlp.down")
        elif ff:
            E, F = ff["router"]["experts"], ff["expert"]["ff"]
            for e in range(E):
                mat(p + f"mlp.e{e}.up", F, D)
                mat(p + f"mlp.e{e}.down", D, F)
                outs.append(p + f"mlp.e{e}.down")
            mat(p + "mlp.router", E, D, std=(0.05 if clear_routes else 1.5) * D ** -0.5)
            w[p + "mlp.router.b"] = bf16((0.02 if clear_routes else 0.5) * rng.standard_normal(E))
            if clear_routes:
                order = np.stack([np.roll(rng.permutation(E), c) for c in range(CLASSES)])
                w[p + "mlp.router"][:, :CLASSES] = bf16(0.25 * order.T)
        mat(p + "side.gate", S, D)
        mat(p + "side.proj", D, S)
        w[p + "side.norm"] = bf16(0.4 + 0.3 * rng.standard_normal(D))
        if clear_routes:
            for name in outs:
                w[name][:CLASSES] = 0.0
    if clear_routes:
        w["embed"][:, :CLASSES] = 6.0 * np.eye(CLASSES)[rng.integers(0, CLASSES, V)]
    return w


def segetar_weights(cfg, seed, clear_routes=True):
    """clear_routes: as for Safolorn, the class's coordinates being taken over from the embedding where a loop mixes the two; one expert
    of every group is corrected upwards, one far down."""
    rng = np.random.default_rng(seed)
    D, V, w, outs = cfg["width"], cfg["vocab"], {}, []

    def mat(name, *shape, std=None):
        w[name] = bf16(rng.standard_normal(shape) * (std or shape[-1] ** -0.5))

    def vec(name, *shape, std=0.2, mean=0.0):
        w[name] = bf16(mean + std * rng.standard_normal(shape))

    def out(name, rows, cols, std=None):
        mat(name, rows, cols, std=std)
        outs.append(name)

    mat("embed", V, D, std=1.0)
    mat("head", V, D)
    vec("final.norm", D, mean=1.0)
    if cfg.get("loop"):
        mat("loop.in", D, 2 * D, std=0.4 * D ** -0.5)
        w["loop.in"] = bf16(w["loop.in"] + np.concatenate([0.8 * np.eye(D), 0.3 * np.eye(D)], axis=1))
        vec("loop.step", cfg["loop"]["times"], D, std=0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x = p + "mix."
        vec(p + "norm1", D, mean=1.0)
        if layer["type"] == "mamba1":
            W, N, R = m["inner"], m["state"], m["dt_rank"]
            mat(x + "in", 2 * W, D)
            mat(x + "conv", W, m["conv"], std=0.6)
            vec(x + "conv.b", W)
            mat(x + "x", R + 2 * N, W)
            mat(x + "dt", W, R, std=0.7 * R ** -0.5)
            vec(x + "dt.b", W, std=1.5, mean=-2.0)
            w[x + "A_log"] = bf16(rng.uniform(-3.0, 2.5, (W, N)))
            vec(x + "D", W, mean=1.0)
            out(x + "o", D, W)
        else:
            l, r, gated = m["left"], m["right"], layer["type"] == "parallel"
            H, G, Hr = l["heads"], l["kv_heads"], r["heads"]
            for name, rows in (("q", H * l["dim"]), ("k", G * l["dim"]), ("v", G * l["vdim"])):
                mat(x + "left." + name, rows, D)
                if gated:
                    vec(x + "left." + name + ".b", rows, std=0.5)
            vec(x + "left.q.norm", H * l["dim"], mean=1.6)
            vec(x + "left.k.norm", G * l["dim"], mean=1.6)
            out(x + "left.o", D, H * l["vdim"])
            for name, rows in (("q", Hr * r["dim"]), ("k", Hr * r["dim"]), ("v", Hr * r["vdim"]), ("g", Hr * r["vdim"])):
                mat(x + "right." + name, rows, D)
            out(x + "right.o", D, Hr * r["vdim"])
            if gated:
                mat(x + "left.g", H, D)
                rank = 3 + i
                mat(x + "right.a1", rank, D)
                mat(x + "right.a2", Hr * r["dim"], rank, std=2.0 * rank ** -0.5)
                vec(x + "right.a2.b", Hr * r["dim"], std=3.0)
                vec(x + "right.norm", r["vdim"], mean=1.0)
            else:
                vec(x + "left.out", D, mean=1.0)
                vec(x + "right.out", D, mean=1.0)
        if not ff:
            continue
        vec(p + "norm2", D, mean=1.0)
        if ff["kind"] == "dense":
            mat(p + "mlp.gate", ff["ff"], D, std=1.5 * D ** -0.5)
            mat(p + "mlp.up", ff["ff"], D)
            out(p + "mlp.down", D, ff["ff"])
            for name, rows in (("gate", ff["ff"]), ("up", ff["ff"]), ("down", D)):
                vec(p + f"mlp.{name}.b", rows)
            outs.append(p + "mlp.down.b")
            continue
        E, F, groups = ff["router"]["experts"], ff["expert"]["ff"], ff["router"]["groups"]["count"]
        for e in range(E):
            mat(p + f"mlp.e{e}.gate", F, D, std=1.5 * D ** -0.5)
            mat(p + f"mlp.e{e}.up", F, D)
            out(p + f"mlp.e{e}.down", D, F)
        mat(p + "mlp.router", E, D, std=(0.02 if clear_routes else 1.5) * D ** -0.5)
        vec(p + "mlp.correction", E, std=0.4)
        if clear_routes:
            # scores of sigmoid(±2.5) at most, by class and rank
            order = np.stack([rng.permutation(E) for _ in range(CLASSES)])
            w[p + "mlp.router"][:, :CLASSES] = bf16((0.8 / E) * (order.T - (E - 1) / 2.0))
            c = np.zeros((groups, E // groups))
            if E // groups > 2:
                c[:, 0], c[:, -1] = -2.0, 0.75
            w[p + "mlp.correction"] = bf16(c.reshape(-1))
            w[p + "norm2"][:CLASSES] = 1.0
    if clear_routes:
        for name in outs:
            w[name][:CLASSES] = 0.0
        w["embed"][:, :CLASSES] = 6.0 * np.eye(CLASSES)[rng.integers(0, CLASSES, V)]
        if cfg.get("loop"):
            w["loop.in"][:CLASSES] = 0.0
            w["loop.in"][:CLASSES, D:D + CLASSES] = np.eye(CLASSES)
            w["loop.step"][:, :CLASSES] = 0.0
    return w


def fororax_weights(cfg, seed, clear_routes=True):
    """clear_routes: as for Safolorn; gains keep the class's coordinates from shrinking as the norms of the sums take their part."""
    rng = np.random.default_rng(seed)
    D, V, w, outs = cfg["width"], cfg["vocab"], {}, []

    def mat(name, *shape, std=None):
        w[name] = bf16(rng.standard_normal(shape) * (std or shape[-1] ** -0.5))

    def vec(name, *shape, std=0.2, mean=0.0):
        w[name] = bf16(mean + std * rng.standard_normal(shape))

    def out(name, rows, cols, std=None):
        mat(name, rows, cols, std=std)
        outs.append(name)

    mat("embed", V, D, std=1.0)
    mat("pos", cfg["max_positions"], D, std=0.6)
    mat("head", V, D, std=2.0 * D ** -0.5)
    vec("final.norm", D, mean=1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x, H, talk = p + "mix.", m["heads"], layer["type"] == "attention_2"
        vec(p + "norm1", D, mean=1.0)
        rows = [("q", H * m["dim"])] + ([("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])] if "kv_from" not in m else [])
        for name, n in rows:
            mat(x + name, n, D)
            if talk:
                vec(x + name + ".b", n, std=0.5)
            if name != "v":
                vec(x + name + ".norm", m["dim"], mean=1.6)
        if talk:
            vec(x + "sink", H, std=1.0, mean=1.0)
            w[x + "talk"] = bf16(0.6 * np.eye(H) + 0.7 * H ** -0.5 * rng.standard_normal((H, H)))
            mat(x + "g", H * m["vdim"], D)
            vec(x + "o.b", D)
            outs.append(x + "o.b")
        else:
            w[x + "r1"], w[x + "r2"] = bf16(rng.uniform(0.2, 1.5, H)), bf16(np.exp(rng.uniform(-5.0, 1.0, H)))
        out(x + "o", D, H * m["vdim"], std=1.5 * (H * m["vdim"]) ** -0.5)
        if not ff:
            continue
        vec(p + "norm2", D, mean=1.0)
        E, n, F, S = ff["router"]["experts"], ff["router"]["experts"] + ff["router"]["identity"], ff["expert"]["ff"], ff["shared"]["ff"]
        for name, width in [(f"e{e}", F) for e in range(E)] + [("shared", S)]:
            mat(p + f"mlp.{name}.gate", width, D, std=1.5 * D ** -0.5)
            mat(p + f"mlp.{name}.up", width, D)
            out(p + f"mlp.{name}.down", D, width)
        mat(p + "mlp.shared.sg", 1, D, std=2.0 * D ** -0.5)
        mat(p + "mlp.router", n, D, std=(0.02 if clear_routes else 1.5) * D ** -0.5)
        vec(p + "mlp.correction", n, std=0.1)
        if clear_routes:
            order = np.stack([rng.permutation(n) for _ in range(CLASSES)])
            w[p + "mlp.router"][:, :CLASSES] = bf16(-0.15 * order.T)
            c = np.zeros(n)
            if n > 4:
                c[rng.integers(n)], c[rng.integers(n)] = -1.0, 1.5
            w[p + "mlp.correction"] = bf16(c)
        for k in ("norm1", "norm2"):
            if clear_routes:
                w[p + k][:CLASSES] = 1.25
    if clear_routes:
        for name in outs:
            w[name][:CLASSES] = 0.0
        w["pos"][:, :CLASSES] = 0.0
        w["embed"][:, :CLASSES] = 4.0 * np.eye(CLASSES)[rng.integers(0, CLASSES, V)]
    return w


def nerenex_weights(cfg, seed):
    rng = np.random.default_rng(seed)
    D, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, *shape, std=None):
        w[name] = bf16(rng.standard_normal(shape) * (std or shape[-1] ** -0.5))

    def vec(name, *shape, std=0.2, mean=0.0):
        w[name] = bf16(mean + std * rng.standard_normal(shape))

    mat("embed", V, D, std=1.0)
    mat("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, D, std=0.7)
    vec("final.norm", D)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        vec(p + "norm1", D)
        mat(p + "rg1", D, D)
        vec(p + "rg1.b", D)
        x = p + "mix."
        if layer["type"] == "latent_attention":
            H = m["heads"]
            mat(x + "dq", m["q_rank"], D)
            vec(x + "dq.norm", m["q_rank"], mean=1.0)
            mat(x + "uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], std=1.6 * m["q_rank"] ** -0.5)
            mat(x + "dkv", m["kv_rank"] + m["rot_dim"], D)
            vec(x + "dkv.norm", m["kv_rank"], mean=1.0)
            mat(x + "uk", H * m["dim"], m["kv_rank"], std=1.6 * m["kv_rank"] ** -0.5)
            mat(x + "uv", H * m["vdim"], m["kv_rank"])
            mat(x + "g", H, D)
            mat(x + "o", D, H * m["vdim"])
        else:
            W, b = m["width"], m["blocks"]
            for n in ("y", "x"):
                mat(x + n, W, D)
                vec(x + n + ".b", W)
            mat(x + "conv", W, m["conv"], std=0.6)
            vec(x + "conv.b", W)
            for n in ("ra", "ri"):
                mat(x + n, b, W // b, W // b)
                vec(x + n + ".b", b, W // b)
            w[x + "lam"] = bf16(rng.uniform(-6.0, 1.0, W))          # decays from almost 1 down to almost 0
            mat(x + "o", D, W)
        if layer["mlp"]:
            F = layer["mlp"]["ff"]
            vec(p + "norm2", D)
            mat(p + "rg2", D, D)
            vec(p + "rg2.b", D)
            mat(p + "mlp.up", F, D, std=2.0 * D ** -0.5)
            mat(p + "mlp.down", D, F)
            w[p + "mlp.act"] = bf16(rng.uniform(-1.0, 1.0, 2))
    return w


def write_checkpoint(path, cfg, w):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, at, blobs = {}, 0, []
    for name, a in w.items():
        assert np.array_equal(bf16(a).reshape(np.shape(a)), np.asarray(a, np.float32)), f"{name} is not bfloat16"
        b = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(b)]}
        at += len(b)
        blobs.append(b)
    h = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return str(path)
