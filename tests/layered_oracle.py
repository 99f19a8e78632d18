"""Plain, slow restatement of the mechanisms layered models are built from (float64 numpy, one function per mechanism).

Test infrastructure: shares no code with the product path.  `forward` walks one sequence from its first token; everything that the
runner carries between portions (latent cache, recurrent state, convolution tail, previous token) is recomputed here from scratch.
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def xielu(z, p, q):
    """Trainable piecewise activation: quadratic right of zero, exponential left of it, slope 1/2 at zero."""
    neg = np.minimum(z, 0.0)
    return np.where(z > 0, softplus(p) * z * z + z / 2, (0.5 + softplus(q)) * (np.expm1(neg) - neg) + z / 2)


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Hash-table row of every token of a sequence; the first token, which has no predecessor, takes the extra row."""
    rows = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return np.array(rows[:len(tokens)], np.int64)


def embed(tokens, table, bigram=None, buckets=0, mul_prev=0, mul_cur=0):
    x = table[np.asarray(tokens)]
    if bigram is not None:
        x = x + bigram[bigram_rows(tokens, buckets, mul_prev, mul_cur)]
    return x


def yarn(dims, base, factor, original, fast, slow):
    """Frequencies of the pairs under YaRN, and the factor of cosines and sines.  A pair that turns more than `fast` times within
    `original` positions keeps its frequency, one that turns less than `slow` times is slowed by `factor`, with a ramp over the pairs
    between them."""
    pair_of = lambda turns: dims * np.log(original / (2.0 * np.pi * turns)) / (2.0 * np.log(base))
    lo, hi = max(np.floor(pair_of(fast)), 0.0), min(np.ceil(pair_of(slow)), dims - 1.0)
    f = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        plain = float(base) ** (-2.0 * i / dims)
        f.append(ramp * plain / factor + (1.0 - ramp) * plain)
    return f, 0.1 * np.log(factor) + 1.0


def rotate_interleaved(x, positions, dims, base, scaling=None):
    """Rotate pairs (2i, 2i + 1) of the first `dims` entries of the last axis; x [tokens, ..., n]."""
    out = x.copy()
    freq, size = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], 1.0
    if scaling:
        freq, size = yarn(dims, base, scaling["factor"], scaling["original"], scaling["fast"], scaling["slow"])
    for i in range(dims // 2):
        a = np.asarray(positions, np.float64) * freq[i]
        c, s = size * np.cos(a), size * np.sin(a)
        shape = (len(c),) + (1,) * (x.ndim - 2)
        c, s = c.reshape(shape), s.reshape(shape)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def window_mask(n, size):
    """[query, key]: a query sees itself and the size − 1 tokens before it."""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < size)


def softmax_attention(scores, mask):
    s = np.where(mask, scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_attention(h, w, heads, dim, rot_dim, vdim, rot_dims, rot_base, window, scale, eps):
    """h [n, width]; w: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o."""
    n = h.shape[0]
    pos = np.arange(n)
    rank = w["dkv"].shape[0] - rot_dim
    q = (unit_rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T
    q = q.reshape(n, heads, dim + rot_dim)
    q_plain, q_rot = q[..., :dim], rotate_interleaved(q[..., dim:], pos, rot_dims, rot_base)
    kv = h @ w["dkv"].T
    latent = unit_rms(kv[:, :rank], eps) * w["dkv.norm"]
    k_rot = rotate_interleaved(kv[:, rank:], pos, rot_dims, rot_base)
    k_plain = (latent @ w["uk"].T).reshape(n, heads, dim)
    value = (latent @ w["uv"].T).reshape(n, heads, vdim)
    mask = window_mask(n, window)
    out = np.zeros((n, heads, vdim))
    for a in range(heads):
        p = softmax_attention((q_plain[:, a] @ k_plain[:, a].T + q_rot[:, a] @ k_rot.T) * scale, mask)
        out[:, a] = p @ value[:, a]
    out *= sigmoid(h @ w["g"].T)[:, :, None]
    return out.reshape(n, heads * vdim) @ w["o"].T


def softmax_with_sink(scores, mask, sink):
    """The sink takes part in the denominator, once, and carries no value."""
    s = np.where(mask, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def latent_and_shared_key(h, w, rank, rot_dims, rot_base, scaling, eps):
    """What a token caches: its normed latent, and the rotated key part that all heads use."""
    kv = h @ w["dkv"].T
    return unit_rms(kv[:, :rank], eps) * w["dkv.norm"], rotate_interleaved(kv[:, rank:], np.arange(h.shape[0]), rot_dims, rot_base, scaling)


def sink_latent_attention(h, w, cached, heads, dim, rot_dim, vdim, rot_dims, rot_base, scaling, scale):
    """Causal attention over `cached` (another layer's, or this one's) with queries straight from h; w: q, uk, uv, sink, o."""
    n = h.shape[0]
    latent, k_rot = cached
    q = (h @ w["q"].T).reshape(n, heads, dim + rot_dim)
    q_plain, q_rot = q[..., :dim], rotate_interleaved(q[..., dim:], np.arange(n), rot_dims, rot_base, scaling)
    k_plain = (latent @ w["uk"].T).reshape(n, heads, dim)
    value = (latent @ w["uv"].T).reshape(n, heads, vdim)
    out = np.zeros((n, heads, vdim))
    for a in range(heads):
        scores = (q_plain[:, a] @ k_plain[:, a].T + q_rot[:, a] @ k_rot.T) * scale
        out[:, a] = softmax_with_sink(scores, window_mask(n, n), w["sink"][a]) @ value[:, a]
    return out.reshape(n, heads * vdim) @ w["o"].T


def causal_conv(x, taps, bias):
    """x [n, c], taps [c, k]: the last column weighs the current token."""
    n, c = x.shape
    k = taps.shape[1]
    padded = np.concatenate([np.zeros((k - 1, c)), x])
    return sum(padded[j:j + n] * taps[:, j] for j in range(k)) + bias


def rglru_scan(u, r, i, lam):
    log_a = -8.0 * r * softplus(lam)
    state, out = np.zeros(u.shape[1]), np.zeros_like(u)
    for t in range(u.shape[0]):
        state = np.exp(log_a[t]) * state + np.sqrt(-np.expm1(2.0 * log_a[t])) * i[t] * u[t]
        out[t] = state
    return out


def block_linear(u, w, b):
    """u [n, blocks·k], w [blocks, k_out, k], b [blocks, k_out]"""
    n, (blocks, ko, k) = u.shape[0], w.shape
    parts = u.reshape(n, blocks, k)
    return np.concatenate([parts[:, j] @ w[j].T + b[j] for j in range(blocks)], axis=1)


def rglru(h, w):
    """w: y, y.b, x, x.b, conv, conv.b, ra, ra.b, ri, ri.b, lam, o."""
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    r, i = sigmoid(block_linear(u, w["ra"], w["ra.b"])), sigmoid(block_linear(u, w["ri"], w["ri.b"]))
    return (rglru_scan(u, r, i, w["lam"]) * y) @ w["o"].T


def dense_ff(h, w):
    """w: up, down, act."""
    return xielu(h @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


def clamped_glu(h, w, limit):
    """w: gate, up, down.  The gate is clamped from above only and turns by a sigmoid of slope 1.702; the linear half is centred at 1."""
    g, u = np.minimum(h @ w["gate"].T, limit), np.clip(h @ w["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def route(logits, top):
    """Experts with the largest logits and the softmax over these logits only."""
    ids = np.argsort(-logits, axis=-1, kind="stable")[:, :top]
    z = np.take_along_axis(logits, ids, axis=-1)
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return ids, e / e.sum(axis=-1, keepdims=True)


def moe(h, w, top):
    """w: router, router.b, e<i>.up, e<i>.down; an expert squares the positive part of its up-projection."""
    ids, weight = route(h @ w["router"].T + w["router.b"], top)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(ids[t], weight[t]):
            out[t] += p * (w[f"e{e}.down"] @ np.maximum(w[f"e{e}.up"] @ h[t], 0.0) ** 2)
    return out


def token_side(x, tokens, w, table, eps):
    """x plus the layer's own view of the token, gated by x; w: gate, proj, norm; table: the layer's columns of the side embedding."""
    return x + unit_rms((gelu_tanh(x @ w["gate"].T) * table[np.asarray(tokens)]) @ w["proj"].T, eps) * w["norm"]


def add_sublayer(x, sub, gate_w, gate_b, norm_w, mult, eps):
    """x + mult · norm(sub · gate): the gate reads x, the norm's weight is stored around zero."""
    gated = sub * sigmoid(x @ gate_w.T + gate_b)
    return x + mult * unit_rms(gated, eps) * (1.0 + norm_w)


def group(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, taps=None):
    """Logits [n, vocab] of one sequence; taps (a list) receives the residual stream after every layer."""
    return {"Nerenex": forward_nerenex, "Safolorn": forward_safolorn, "Segetar": forward_segetar,
            "Fororax": forward_fororax}[config["architecture"]](config, weights, tokens, taps)

def silu(z):
    return z * sigmoid(z)


def rotated_halves(x, positions, dims, base):
    """Rotate pairs (i, i + dims/2) of the first `dims` entries of the last axis; x [tokens, ..., n]."""
    out, half = x.copy(), dims // 2
    for i in range(half):
        a = np.asarray(positions, np.float64) * float(base) ** (-2.0 * i / dims)
        shape = (len(a),) + (1,) * (x.ndim - 2)
        c, s = np.cos(a).reshape(shape), np.sin(a).reshape(shape)
        u, v = x[..., i], x[..., half + i]
        out[..., i] = u * c - v * s
        out[..., half + i] = v * c + u * s
    return out


def grouped_attention(h, w, heads, kv_heads, dim, vdim, window, scale, eps, rot=None):
    """Sliding-window attention with shared key / value heads; queries and keys are normed over all their rows at once.  w: q, k, v
    (with q.b, k.b, v.b: biases), q.norm, k.norm, o (with g: a sigmoid gate per head); rot: (dims, base), interleaved pairs."""
    n, pos = h.shape[0], np.arange(h.shape[0])
    lin = lambda name: h @ w[name].T + w.get(name + ".b", 0.0)
    q = (unit_rms(lin("q"), eps) * w["q.norm"]).reshape(n, heads, dim)
    k = (unit_rms(lin("k"), eps) * w["k.norm"]).reshape(n, kv_heads, dim)
    v = lin("v").reshape(n, kv_heads, vdim)
    if rot:
        q, k = rotate_interleaved(q, pos, *rot), rotate_interleaved(k, pos, *rot)
    mask, out = window_mask(n, window), np.zeros((n, heads, vdim))
    for a in range(heads):
        g = a // (heads // kv_heads)
        out[:, a] = softmax_attention((q[:, a] @ k[:, g].T) * scale, mask) @ v[:, g]
    if "g" in w:
        out *= sigmoid(h @ w["g"].T)[:, :, None]
    return out.reshape(n, heads * vdim) @ w["o"].T


def decayed_state(q, k, v, decay):
    """Per head S_t = diag(decay_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; q, k, decay [n, heads, dim], v [n, heads, vdim]."""
    n, heads, dim = q.shape
    state, out = np.zeros((heads, dim, v.shape[2])), np.zeros(v.shape)
    for t in range(n):
        state = decay[t][:, :, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hd,hdv->hv", q[t], state)
    return out


def gated_linear_attention(h, w, heads, dim, vdim, tau, eps):
    """w: q, k, v, g, o, norm, a1, a2, a2.b.  The decay of a key channel is read from the input through a narrow projection."""
    n = h.shape[0]
    q, k = (h @ w["q"].T * dim ** -0.5).reshape(n, heads, dim), (h @ w["k"].T).reshape(n, heads, dim)
    v = (h @ w["v"].T).reshape(n, heads, vdim)
    decay = sigmoid((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]) ** (1.0 / tau)
    o = unit_rms(decayed_state(q, k, v, decay.reshape(n, heads, dim)), eps) * w["norm"]
    return (o.reshape(n, heads * vdim) * silu(h @ w["g"].T)) @ w["o"].T


def retention(h, w, heads, dim, vdim, decay, rot, eps):
    """w: q, k, v, g, o; a constant decay per head, rotated queries and keys, heads' results over their root mean square."""
    n, pos = h.shape[0], np.arange(h.shape[0])
    q = rotated_halves((h @ w["q"].T).reshape(n, heads, dim), pos, *rot)
    k = rotated_halves((h @ w["k"].T).reshape(n, heads, dim), pos, *rot) * dim ** -0.5
    v = (h @ w["v"].T).reshape(n, heads, vdim)
    d = np.broadcast_to(np.asarray(decay, np.float64)[None, :, None], (n, heads, dim))
    return (unit_rms(decayed_state(q, k, v, d), eps).reshape(n, heads * vdim) * silu(h @ w["g"].T)) @ w["o"].T


def selective_scan(h, w, inner, dt_rank, state):
    """w: in, conv, conv.b, x, dt, dt.b, A_log, D, o."""
    xz = h @ w["in"].T
    x, z = silu(causal_conv(xz[:, :inner], w["conv"], w["conv.b"])), xz[:, inner:]
    low = x @ w["x"].T
    dt = softplus(low[:, :dt_rank] @ w["dt"].T + w["dt.b"])
    b, c = low[:, dt_rank:dt_rank + state], low[:, dt_rank + state:]
    a, s, y = -np.exp(w["A_log"]), np.zeros((inner, state)), np.zeros(x.shape)
    for t in range(len(h)):
        s = np.exp(dt[t][:, None] * a) * s + (dt[t] * x[t])[:, None] * b[t][None, :]
        y[t] = s @ c[t] + w["D"] * x[t]
    return (y * silu(z)) @ w["o"].T


def gelu_glu(h, w):
    """w: gate, gate.b, up, up.b, down, down.b."""
    return (gelu_tanh(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])) @ w["down"].T + w["down.b"]


def grouped_route(logits, correction, top, groups, keep, scale):
    """Experts and weights of one token.  The correction takes part in the choice only; a group counts by its two best choices, and
    experts outside the best `keep` groups cannot be chosen."""
    s = sigmoid(logits)
    choice = (s + correction).reshape(groups, -1)
    rank = np.sort(choice, axis=1)[:, -2:].sum(axis=1)
    out = np.ones(groups, bool)
    out[np.argsort(-rank, kind="stable")[:keep]] = False
    choice[out] = -np.inf
    ids = np.argsort(-choice.reshape(-1), kind="stable")[:top]
    return ids, s[ids] / (s[ids].sum() + 1e-20) * scale


def silu_moe(h, w, top, groups, keep, scale):
    """w: router, correction, e<i>.gate, e<i>.up, e<i>.down."""
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(*grouped_route(w["router"] @ h[t], w["correction"], top, groups, keep, scale)):
            out[t] += p * (w[f"e{e}.down"] @ (silu(w[f"e{e}.gate"] @ h[t]) * (w[f"e{e}.up"] @ h[t])))
    return out


def segetar_mixer(h, layer, w, eps):
    m = layer["mixer"]
    if layer["type"] == "mamba1":
        return selective_scan(h, w, m["inner"], m["dt_rank"], m["state"])
    l, r = m["left"], m["right"]
    rot = lambda x: (x["rot"]["dims"], x["rot"]["base"])
    left = grouped_attention(h, group(w, "left."), l["heads"], l["kv_heads"], l["dim"], l["vdim"], l["mask"]["size"], l["scale"], eps,
                             rot(l) if layer["type"] == "parallel" else None)
    rw = group(w, "right.")
    if layer["type"] == "parallel":
        return m["left_scale"] * left + m["right_scale"] * gated_linear_attention(h, rw, r["heads"], r["dim"], r["vdim"], r["tau"], eps)
    right = retention(h, rw, r["heads"], r["dim"], r["vdim"], r["decay"], rot(r), eps)
    return (unit_rms(left, eps) * w["left.out"] + unit_rms(right, eps) * w["right.out"]) / 2


def layer_runs(config):
    """(layer, pass) in the order they run; pass −1: outside the loop."""
    n, lp = len(config["layers"]), config.get("loop")
    if not lp:
        return [(i, -1) for i in range(n)]
    return ([(i, -1) for i in range(lp["start"])] + [(i, t) for t in range(lp["times"]) for i in range(lp["start"], lp["stop"])]
            + [(i, -1) for i in range(lp["stop"], n)])


def forward_segetar(config, weights, tokens, taps=None):
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x0 = embed(tokens, w["embed"])
    x = x0
    for li, t in layer_runs(config):
        layer, p = config["layers"][li], f"l{li}."
        if t >= 0 and li == config["loop"]["start"]:
            x = np.concatenate([x, x0], axis=1) @ w["loop.in"].T + w["loop.step"][t]
        x = x + segetar_mixer(unit_rms(x, eps) * w[p + "norm1"], layer, group(w, p + "mix."), eps)
        ff = layer["mlp"]
        if ff:
            h, fw = unit_rms(x, eps) * w[p + "norm2"], group(w, p + "mlp.")
            if ff["kind"] == "dense":
                x = x + gelu_glu(h, fw)
            else:
                r = ff["router"]
                x = x + silu_moe(h, fw, r["top"], r["groups"]["count"], r["groups"]["keep"], r["scale"])
        if taps is not None:
            taps.append(x.copy())
    return (unit_rms(x, eps) * w["final.norm"]) @ w["head"].T


def embed_at_positions(tokens, table, factor, positions):
    """The token's row times a factor plus the row of its position, which is not scaled."""
    return table[np.asarray(tokens)] * factor + positions[:len(tokens)]


def head_normed(x, heads, gain, eps):
    """[n, heads·dim] → [n, heads, dim], every head over its own root mean square, times one gain for all of them."""
    return unit_rms(x.reshape(x.shape[0], heads, -1), eps) * gain


def log_distance(n, r1, r2):
    """[query, key]: what is taken off a score, growing with the logarithm of the distance (future keys: 0, they are masked)."""
    return r1 * np.log1p(r2 * np.maximum(np.arange(n)[:, None] - np.arange(n)[None, :], 0))


def keys_and_values(h, w, kv_heads, vdim, eps):
    """What a token caches; w: k, k.norm, v (with k.b, v.b: biases)."""
    lin = lambda name: h @ w[name].T + w.get(name + ".b", 0.0)
    return head_normed(lin("k"), kv_heads, w["k.norm"], eps), lin("v").reshape(h.shape[0], kv_heads, vdim)


def log_distance_attention(h, w, cached, heads, scale, eps):
    """Causal attention whose scores lose r1 ln(1 + r2 distance); `cached`: keys and values of this layer or an earlier one; w: q, q.norm, r1,
    r2, o."""
    n, (k, v) = h.shape[0], cached
    q, share = head_normed(h @ w["q"].T, heads, w["q.norm"], eps), heads // k.shape[1]
    out = np.zeros((n, heads, v.shape[2]))
    for a in range(heads):
        scores = (q[:, a] @ k[:, a // share].T) * scale - log_distance(n, w["r1"][a], w["r2"][a])
        out[:, a] = softmax_attention(scores, window_mask(n, n)) @ v[:, a // share]
    return out.reshape(n, -1) @ w["o"].T


def mix_heads(weights, talk):
    """[heads, query, key]: every head's weights become a mixture of all heads' weights."""
    return np.einsum("hg,gij->hij", talk, weights)


def talking_attention(h, w, cached, heads, scale, eps):
    """Causal attention with sinks whose heads' weights are mixed between softmax and values, with a gate per value element; w: q, q.b, q.norm,
    sink, talk, g, o, o.b."""
    n, (k, v) = h.shape[0], cached
    q, share = head_normed(h @ w["q"].T + w["q.b"], heads, w["q.norm"], eps), heads // k.shape[1]
    p = np.stack([softmax_with_sink((q[:, a] @ k[:, a // share].T) * scale, window_mask(n, n), w["sink"][a]) for a in range(heads)])
    p = mix_heads(p, w["talk"])
    out = np.stack([p[a] @ v[:, a // share] for a in range(heads)], axis=1).reshape(n, -1)
    return (out * sigmoid(h @ w["g"].T)) @ w["o"].T + w["o.b"]


def corrected_softmax_route(logits, correction, top):
    """Experts and weights of one token: softmax over all of them; the correction takes part in the choice only, and the weights stay the
    chosen scores as they are."""
    e = np.exp(logits - logits.max())
    s = e / e.sum()
    ids = np.argsort(-(s + correction), kind="stable")[:top]
    return ids, s[ids]


def identity_moe(h, w, experts, top, limit):
    """w: router, correction, e<i>.gate, e<i>.up, e<i>.down.  Experts from number `experts` on hand their input on."""
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(*corrected_softmax_route(w["router"] @ h[t], w["correction"], top)):
            out[t] += p * (clamped_glu(h[t:t + 1], group(w, f"e{e}."), limit)[0] if e < experts else h[t])
    return out


def gated_shared_expert(h, w, limit):
    """w: gate, up, down, sg: one factor per token."""
    return clamped_glu(h, w, limit) * sigmoid(h @ w["sg"].T)


def softcap(logits, cap):
    return cap * np.tanh(logits / cap)


def forward_fororax(config, weights, tokens, taps=None):
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    eps, alpha = config["norm"]["eps"], config["postln_alpha"]
    x, cached = embed_at_positions(tokens, w["embed"], config["embedding"]["scale"], w["pos"]), {}
    for li, layer in enumerate(config["layers"]):
        p, m, ff = f"l{li}.", layer["mixer"], layer["mlp"]
        mw, src = group(w, p + "mix."), m.get("kv_from", li)
        if src == li:
            cached[li] = keys_and_values(x, mw, m["kv_heads"], m["vdim"], eps)
        mixer = log_distance_attention if layer["type"] == "attention" else talking_attention
        x = unit_rms(alpha * x + mixer(x, mw, cached[src], m["heads"], m["scale"], eps), eps) * w[p + "norm1"]
        if ff:
            fw, r = group(w, p + "mlp."), ff["router"]
            y = identity_moe(x, fw, r["experts"], r["top"], ff["expert"]["limit"]) + gated_shared_expert(x, group(fw, "shared."), ff["shared"]["limit"])
            x = unit_rms(alpha * x + y, eps) * w[p + "norm2"]
        if taps is not None:
            taps.append(x.copy())
    return softcap((unit_rms(x, eps) * w["final.norm"]) @ w["head"].T, config["logit_softcap"])


def forward_safolorn(config, weights, tokens, taps=None):
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    eps, side = config["norm"]["eps"], config["token_side"]["dim"]
    x = embed(tokens, w["embed"])
    cached = {}
    for li, layer in enumerate(config["layers"]):
        p, mx, ff = f"l{li}.", layer["mixer"], layer["mlp"]
        mw, rot = group(w, p + "mix."), mx["rot"]
        xhat = unit_rms(x, eps)
        h = xhat * w[p + "norm1"]
        if "kv_from" not in mx:
            cached[li] = latent_and_shared_key(h, mw, mx["kv_rank"], rot["dims"], rot["base"], rot.get("scaling"), eps)
        y = sink_latent_attention(h, mw, cached[mx.get("kv_from", li)], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], rot["dims"],
                                  rot["base"], rot.get("scaling"), mx["scale"])
        if ff:
            h2, fw = xhat * w[p + "norm2"], group(w, p + "mlp.")
            y = y + (clamped_glu(h2, fw, ff["limit"]) if ff["kind"] == "dense" else moe(h2, fw, ff["router"]["top"]))
        x = token_side(x + y, tokens, group(w, p + "side."), w["side.embed"][:, li * side:(li + 1) * side], eps)
        if taps is not None:
            taps.append(x.copy())
    return (unit_rms(x, eps) * w["final.norm"]) @ w["head"].T


def forward_nerenex(config, weights, tokens, taps=None):
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    bg = config["embedding"]["bigram"]
    x = embed(tokens, w["embed"], w["bigram"], bg["buckets"], bg["mul_prev"], bg["mul_cur"])
    for li, layer in enumerate(config["layers"]):
        p, mx = f"l{li}.", layer["mixer"]
        mw = group(w, p + "mix.")
        if layer["type"] == "latent_attention":
            sub = latent_attention(x, mw, mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["rot"]["dims"], mx["rot"]["base"],
                                   mx["mask"]["size"], mx["scale"], eps)
        else:
            sub = rglru(x, mw)
        x = add_sublayer(x, sub, w[p + "rg1"], w[p + "rg1.b"], w[p + "norm1"], mult, eps)
        if layer["mlp"]:
            x = add_sublayer(x, dense_ff(x, group(w, p + "mlp.")), w[p + "rg2"], w[p + "rg2.b"], w[p + "norm2"], mult, eps)
        if taps is not None:
            taps.append(x.copy())
    return (unit_rms(x, eps) * (1.0 + w["final.norm"])) @ w["embed"].T


def greedy(config, weights, prompt, steps):
    out, seq = [], list(prompt)
    for _ in range(steps):
        t = int(np.argmax(forward(config, weights, seq)[-1]))
        out.append(t)
        seq.append(t)
    return out
