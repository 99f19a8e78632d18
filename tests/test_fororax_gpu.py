"""Fororax's mechanisms on the device against the plain oracle of tests/layered_oracle.py: each alone through the taps of small models,
with mistakes planted in the oracle where random weights would hide them; whole models, batches and the engine loop are covered with
the other layered architectures in test_layered_gpu.py."""
import json

import numpy as np
import pytest

from tests import layered_gen as G
from tests import layered_oracle as L
from tests.test_layered_gpu import DTYPES, TOL, cases, feed, load, pkg, rel, taps_of, toks  # noqa: F401  (two are fixtures)

pytestmark = pytest.mark.gpu
ALONE = {"float32": 1e-5, "bfloat16": 2e-2}


def model(layers, width=72, vocab=50, alpha=0.5, **kw):
    return G.fororax(width, vocab, layers, alpha=alpha, **kw)


def changed(cfg, edit):
    c = json.loads(json.dumps(cfg))
    edit(c)
    return c


def silence(w, *what):
    for k in w:
        if k.split(".", 1)[-1] in what:
            w[k][:] = 0.0


def agree(pkg, tmp_path, cfg, w, dtype, n=70, tol=None, seed=6):
    t, taps = toks(cfg, n, seed), []
    L.forward(cfg, w, t, taps)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t), taps) < (tol or ALONE[dtype])
    return t, taps


def differs(cfg, w, t, taps, bound=1e-3):
    other = []
    L.forward(cfg, w, t, other)
    return rel(other, taps) > bound


# ── embedding, norm of the sum, capped logits ─────────────────────────────────────────────────────────────────────────────
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,factor", [(72, 2.5), (45, 0.3), (33, 1.0)])
def test_scaled_embedding_and_positions_across_portions(pkg, tmp_path, dtype, width, factor):
    """A layer that adds nothing: the stream is the normed embedding, with the position's vector outside the factor, counted on over portions,
    decode steps and in a sequence that takes over another one's pages."""
    cfg = model([G.far_attention(2, 1, 8, 8)], width=width, scale=factor, positions=40)
    w = G.weights(cfg, 3, clear_routes=False)
    silence(w, "mix.o")
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=40, seqs=2, blocks=3)
    m.enable_taps()
    t, taps = toks(cfg, 40, 5), []
    L.forward(cfg, w, t, taps)
    assert differs(changed(cfg, lambda c: c["embedding"].update(scale=factor + 0.2)), w, t, taps, 1e-2)
    for seq, cuts in ((1, [40]), (2, [1, 2, 7, 1, 16]), (3, [15, 1, 1, 4, 1])):
        at = 0
        while at < len(t):
            n = min(cuts.pop(0) if cuts else 3, len(t) - at)
            m.forward_rows([(seq, t[at:at + n], at)], [])
            assert np.abs(m.read_taps(n)[0] - taps[0][at:at + n]).max() < 1e-5
            at += n
        m.release(seq)
    with pytest.raises(RuntimeError, match="max_seq_len"):
        m.forward_rows([(9, toks(cfg, 41, 5), 0)], [])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("alpha,eps", [(1.0, 1e-6), (3.0, 1e-5), (0.25, 0.4), (7.0, 2.0)])
def test_norm_of_the_sum(pkg, tmp_path, dtype, alpha, eps):
    """The factor of the stream on both sublayers, a large epsilon, a layer without feed-forward."""
    cfg = model([G.talk_attention(2, 1, 16, 16, mlp=G.identity_experts(3, 1, 2, 24, 20)), G.far_attention(2, 2, 12, 8)], alpha=alpha, eps=eps)
    w = G.weights(cfg, 5)
    t, taps = agree(pkg, tmp_path, cfg, w, dtype)
    assert differs(changed(cfg, lambda c: c.update(postln_alpha=alpha * 1.1)), w, t, taps, 1e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cap", [0.5, 4.0, 300.0])
def test_capped_logits(pkg, tmp_path, dtype, cap):
    cfg = model([G.far_attention(2, 1, 16, 16)], cap=cap, vocab=77)
    w, t = G.weights(cfg, 7), toks(model([]), 30, 8)
    w["head"] *= 4.0
    want = L.forward(cfg, w, t)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    got = feed(m, 1, t, [20, 1])
    assert rel(got, want) < TOL[dtype] and np.abs(got).max() <= cap * 1.0001
    assert (rel(L.forward(changed(cfg, lambda c: c.update(logit_softcap=1e9)), w, t), want) > 0.1) == (cap < 100)


# ── attention ─────────────────────────────────────────────────────────────────────────────────────────────────────────────
FAR = [G.far_attention(4, 2, 20, 28), G.far_attention(6, 1, 32, 32, scale=0.4), G.far_attention(5, 5, 7, 3), G.far_attention(40, 2, 64, 48), G.far_attention(3, 3, 100, 130),
       G.far_attention(2, 1, 260, 40), G.far_attention(9, 3, 180, 96, scale=0.03)]
TALK = [G.talk_attention(4, 2, 20, 28), G.talk_attention(6, 3, 32, 32, scale=0.4), G.talk_attention(1, 1, 5, 3), G.talk_attention(24, 8, 64, 40), G.talk_attention(7, 7, 100, 130),
        G.talk_attention(2, 1, 260, 40), G.talk_attention(16, 16, 40, 96, scale=0.2), G.talk_attention(20, 5, 128, 128), G.talk_attention(17, 1, 32, 32), G.talk_attention(32, 16, 48, 64),
        G.talk_attention(40, 4, 24, 24), G.talk_attention(3, 1, 200, 256), G.talk_attention(30, 10, 90, 20), G.talk_attention(12, 12, 33, 64)]
FORMS = {"plain": dict(GROUPED_PLAIN=1), "keys": dict(GROUPED_SPLITS=1, GROUPED_TILE_MIN_ROWS=10 ** 6, TALK_TILE_MIN_TOKENS=0),
         "split": dict(GROUPED_SPLITS=4, GROUPED_TILE_MIN_ROWS=10 ** 6, TALK_TILE_MIN_TOKENS=0), "tile": dict(GROUPED_SPLITS=1, GROUPED_TILE_MIN_ROWS=1, TALK_TILE_MIN_TOKENS=1, TALK_TILE_SPLITS=1),
         "tile split": dict(GROUPED_SPLITS=1, GROUPED_TILE_MIN_ROWS=1, TALK_TILE_MIN_TOKENS=1, TALK_TILE_SPLITS=3)}
CASES = [("plain", "float32")] + [(f, "bfloat16") for f in FORMS]


@pytest.mark.parametrize("form,dtype", CASES[:-1])
@pytest.mark.parametrize("i", range(len(FAR)))
def test_far_attention_alone(pkg, tmp_path, knobs, forms, form, dtype, i):
    knobs.set(**FORMS[form])
    cfg = model([FAR[i]])
    w = G.weights(cfg, 20 + i)
    forms.reset()
    t, taps = agree(pkg, tmp_path, cfg, w, dtype, tol=ALONE[dtype] * (1 if dtype == "float32" else 2))
    big = max(FAR[i]["mixer"]["dim"], FAR[i]["mixer"]["vdim"]) > 256
    assert forms.hits().get("grouped_attn_plain" if big else {"plain": "grouped_attn_plain", "keys": "grouped_attn_keys", "split": "grouped_attn_split", "tile": "grouped_attn_tile"}[form])
    for k in ("r1", "r2"):
        wrong = dict(w)
        wrong["l0.mix." + k] = w["l0.mix." + k] * np.float32(1.2)
        assert differs(cfg, wrong, t, taps)
    wrong = dict(w)                                                             # gains are of the head's dimensions, the mean square one head's own
    wrong["l0.mix.q.norm"] = np.roll(w["l0.mix.q.norm"], 1)
    assert differs(cfg, wrong, t, taps)


@pytest.mark.parametrize("form,dtype", CASES)
@pytest.mark.parametrize("i", range(len(TALK)))
def test_talking_attention_alone(pkg, tmp_path, knobs, forms, form, dtype, i):
    knobs.set(**FORMS[form])
    cfg = model([TALK[i]])
    w = G.weights(cfg, 40 + i)
    forms.reset()
    t, taps = agree(pkg, tmp_path, cfg, w, dtype, tol=ALONE[dtype] * (1 if dtype == "float32" else 2))
    m, h = TALK[i]["mixer"], forms.hits()
    if form == "plain" or m["heads"] > 32 or max(m["dim"], m["vdim"]) > (256 if m["heads"] <= 16 else 128):
        assert h.get("talk_attn_plain")
    elif "tile" in form or m["kv_heads"] > (8 if m["heads"] > 16 or max(m["dim"], m["vdim"]) > 128 else 16) or m["heads"] // m["kv_heads"] > 16:
        assert h.get("talk_attn_tile") and not h.get("talk_attn_plain") and bool(h.get("talk_attn_tile_split")) == ("split" in form and "tile" in form)
    else:
        assert h.get("talk_attn_keys") and not h.get("talk_attn_tile")
    H = m["heads"]
    for name, new in (("talk", w["l0.mix.talk"].T if H > 1 else 2 * w["l0.mix.talk"]), ("sink", w["l0.mix.sink"] - 1), ("k.b", 0 * w["l0.mix.k.b"] + 1), ("o.b", 0 * w["l0.mix.o.b"]),
                      ("g", w["l0.mix.g"] * 2), ("v.b", w["l0.mix.v.b"] + np.float32(0.5))):
        wrong = dict(w)
        wrong["l0.mix." + name] = np.asarray(new, np.float32)
        assert differs(cfg, wrong, t, taps), name


@pytest.mark.parametrize("form,dtype", CASES)
def test_prompts_portions_and_decoding_of_long_contexts(pkg, tmp_path, knobs, form, dtype):
    """Several key splits and many steps per tile; portions that start anywhere in a page, single tokens in between; scattered pages."""
    knobs.set(**FORMS[form])
    cfg = model([G.talk_attention(12, 4, 32, 32), G.far_attention(6, 2, 32, 32), G.talk_attention(20, 4, 64, 64), G.far_attention(6, 2, 32, 32, kv_from=1)], alpha=1.0, positions=800)
    w, t = G.weights(cfg, 71), toks(cfg, 700, 72)
    want = L.forward(cfg, w, t)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=1600, max_len=800)
    m.forward_rows([(90, t[:33], 0), (91, t[:50], 0)], [])
    m.release(90)
    for i, cuts in enumerate(([700], [650, 1, 1, 1, 13, 2, 1], [31, 17, 128, 2, 300, 1, 64], [513, 180, 7])):
        assert rel(feed(m, i, t, cuts), want) < TOL[dtype], cuts
        m.release(i)
    knobs.set(GROUPED_SPLITS=50)                                                # more splits than some tokens have steps
    assert rel(feed(m, 9, t, [690, 3, 1]), want) < TOL[dtype]


def standout(kind, heads=6, kv_heads=2, dim=32, vdim=32, score=24.0, seed=5, sink=2.0):
    """One attention layer in which token 1's query scores token 0's key far above every other key, wherever they are."""
    layer = (G.talk_attention if kind == "talk" else G.far_attention)(heads, kv_heads, dim, vdim, scale=score / dim)
    cfg = model([layer], vocab=60)
    w = G.weights(cfg, seed, clear_routes=False)
    w["pos"][:] = 0.0
    p = "l0.mix."
    w[p + "q.norm"][:] = 1.0
    w[p + "k.norm"][:] = 1.0
    if kind == "talk":
        for b in ("q.b", "k.b"):
            w[p + b][:] = 0.0
        w[p + "sink"][:] = sink
    else:
        w[p + "r1"][:], w[p + "r2"][:] = 0.5, 0.25
    e = w["embed"].astype(np.float64)
    k = (w[p + "k"].astype(np.float64) @ e[0]).reshape(kv_heads, dim)
    q = np.concatenate([np.outer(k[a * kv_heads // heads] / np.linalg.norm(k[a * kv_heads // heads]), e[1] / np.linalg.norm(e[1])) for a in range(heads)])
    w[p + "q"] = G.bf16(q + 0.01 * w[p + "q"])
    return cfg, w


@pytest.mark.parametrize("form,dtype", CASES)
@pytest.mark.parametrize("kind,sizes", [("far", {}), ("talk", {}), ("talk", dict(heads=24, kv_heads=4)), ("talk", dict(heads=8, kv_heads=8, dim=64, vdim=64))])
def test_far_key_and_future_key(pkg, tmp_path, knobs, form, dtype, kind, sizes):
    """The key that stands out sits hundreds of tokens back, at a page border, in a prompt, a portion of two and decoded; standing right
    behind the query it must not be seen."""
    knobs.set(**FORMS[form])
    cfg, w = standout(kind, **sizes)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=512)
    seq = 0
    for at, back in ((0, 1), (15, 290), (16, 290), (17, 63), (31, 64), (32, 400), (0, 447)):
        t = toks(cfg, at + back + 3, 80) % 50 + 5
        q = at + back
        t[at], t[q], t[q + 1] = 0, 1, 0                                       # the same token right behind the query
        blind = t.copy()
        blind[at] = 7
        want, none = L.forward(cfg, w, t)[q], L.forward(cfg, w, blind)[q]
        assert rel(none[None], want[None]) > 3 * TOL["bfloat16"]
        for tokens, ref in ((t, want), (blind, none)):
            for cuts in ([len(t)], [q, 1, 1], [max(1, q - 1), 2, 1], [max(1, q), 2], [40, 100, 65]):
                assert rel(feed(m, seq, tokens, cuts)[q:q + 1], ref[None]) < TOL[dtype], (at, back, cuts)
                m.release(seq)
                seq += 1


@pytest.mark.parametrize("form,dtype", CASES)
@pytest.mark.parametrize("sink", [-60.0, 0.0, 24.0, 120.0])
def test_sink_against_scores(pkg, tmp_path, knobs, form, dtype, sink):
    """A sink far below, among, level with the best score, and far above every score (the heads then add nothing, mixed or not)."""
    knobs.set(**FORMS[form])
    cfg, w = standout("talk", sink=sink)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=256)
    t = toks(cfg, 190, 81) % 50 + 5
    t[3], t[189], t[70] = 0, 1, 1
    want = L.forward(cfg, w, t)
    without = dict(w)
    without["l0.mix.sink"] = np.full(6, -1e9, np.float32)
    assert (rel(L.forward(cfg, without, t)[-1:], want[-1:]) > 3 * TOL["bfloat16"]) == (sink > 10)
    for i, cuts in enumerate(([190], [188, 1], [100, 64, 2], [1, 1, 1, 187])):
        assert rel(feed(m, i, t, cuts), want) < TOL[dtype], cuts
        m.release(i)


@pytest.mark.parametrize("form,dtype", CASES)
def test_one_head_speaks_through_another(pkg, tmp_path, knobs, form, dtype):
    """Head 0 sees the key that stands out and says nothing itself; its weights reach the values of a head of another key / value head, with a
    negative factor, and a wide mixture of large opposite factors cancels."""
    knobs.set(**FORMS[form])
    cfg, w = standout("talk")
    T = np.zeros((6, 6))
    T[5, 0], T[2] = -1.5, [8.0, -8.0, 8.0, -8.0, 8.0, -8.0]
    w["l0.mix.talk"] = G.bf16(T)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=256)
    t = toks(cfg, 190, 83) % 50 + 5
    t[40], t[189] = 0, 1
    want = L.forward(cfg, w, t)
    for i, cuts in enumerate(([190], [189, 1], [100, 88, 2])):
        assert rel(feed(m, i, t, cuts)[-1:], want[-1:]) < TOL[dtype], cuts
        m.release(i)


@pytest.mark.parametrize("form,dtype", CASES)
@pytest.mark.parametrize("window", [1, 2, 16, 17, 64, 100])
def test_windows_of_talking_attention(pkg, tmp_path, knobs, form, dtype, window):
    """The mechanism takes a window like the other grouped attention; the key that stands out is on its edge, or one further back."""
    knobs.set(**FORMS[form])
    cfg, w = standout("talk", heads=8, kv_heads=2)
    d, _, _ = pkg.Checkpoint(G.write_checkpoint(tmp_path, cfg, w)).model_config(300)
    lc, specs = pkg.Checkpoint(str(tmp_path)).layered_config()
    specs[0].window = window
    lc.dtype = 1 if dtype == "float32" else 0
    m = pkg.HipModel(layered=(lc, specs), **{**d, "max_seq_len": 300, "kv_num_blocks": 40, "max_seqs": 4, "max_tokens": 300})
    for k, v in w.items():
        m.set_tensor(k, v)
    m.finalize()
    oracle, mask = L.window_mask, lambda n, size: np.abs(np.subtract.outer(np.arange(n), np.arange(n)) - (window - 1) / 2) <= (window - 1) / 2
    seq = 0
    for at in (0, 3, 15, 16):
        for back in (window - 1, window):
            t = toks(cfg, at + back + 1, 70) % 50 + 5
            t[at] = 0 if back else 1
            t[at + back] = 1
            try:
                L.window_mask = mask
                want = L.forward(cfg, w, t)[-1:]
            finally:
                L.window_mask = oracle
            if back == window:
                assert rel(L.forward(cfg, w, t)[-1:], want) > 3 * TOL["bfloat16"]
            for cuts in ([len(t)], [max(1, len(t) - 1), 1], [max(1, len(t) - 2), 2], [max(1, len(t) - 3), 2, 1]):
                assert rel(feed(m, seq, t, cuts)[-1:], want) < TOL[dtype], (at, back, cuts)
                m.release(seq)
                seq += 1


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[70], [1], [40, 3, 2, 1], [20, 50]])
def test_keys_of_an_earlier_layer(pkg, tmp_path, dtype, cuts):
    """Layers 2 to 4 read what layers 0 and 1 have cached, in this portion and in earlier ones, with queries, distances and head counts of their
    own."""
    cfg = model([G.far_attention(4, 2, 16, 20), G.far_attention(3, 3, 24, 12), G.far_attention(6, 2, 16, 20, kv_from=0), G.far_attention(3, 3, 24, 12, kv_from=1),
                 G.far_attention(2, 2, 16, 20, kv_from=0)], alpha=1.5)
    w, t = G.weights(cfg, 53), toks(cfg, 70, 6)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    want = L.forward(cfg, w, t)
    assert rel(feed(m, 1, t, cuts), want) < TOL[dtype]
    own = changed(cfg, lambda c: c["layers"][2]["mixer"].pop("kv_from"))
    ow = dict(w)
    for k in ("k", "v", "k.norm"):
        ow["l2.mix." + k] = w["l0.mix." + k]
    assert rel(L.forward(own, ow, t), want) > 3 * TOL[dtype]                   # (the same projections of another layer's input)


# ── experts ───────────────────────────────────────────────────────────────────────────────────────────────────────────────
def experts_only(mlp, seed, clear, width=72):
    """A layer whose mixer adds nothing; the stream is then the normed embedding."""
    cfg = model([G.far_attention(1, 1, 8, 8, mlp=mlp)], width=width)
    w = G.weights(cfg, seed, clear_routes=clear)
    silence(w, "mix.o")
    return cfg, w


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,identity,top,ff,shared", [(7, 3, 3, 41, 50), (16, 0, 1, 64, 33), (5, 3, 8, 20, 90), (1, 1, 1, 33, 1), (1, 0, 1, 9, 16), (2, 9, 3, 24, 24), (60, 10, 6, 24, 40),
                                                      (100, 30, 2, 40, 20), (250, 60, 7, 9, 12)])
@pytest.mark.parametrize("tokens", [1, 3, 90, 200])
def test_experts_alone(pkg, tmp_path, forms, dtype, n, identity, top, ff, shared, tokens):
    """Routing and sorting in one launch and in two, on every number of experts per lane; identity experts in any share of the choices, all of
    them included; 32-bit: routers that read everything."""
    cfg, w = experts_only(G.identity_experts(n, identity, top, ff, shared, 0.9, 1.7), 43, dtype == "bfloat16")
    forms.reset()
    t, taps = agree(pkg, tmp_path, cfg, w, dtype, n=tokens)
    h = forms.hits()
    assert bool(h.get("moe_route_sort")) == (tokens * top <= 1024) and bool(h.get("route_softmax")) == (tokens * top > 1024)
    if dtype == "float32":
        wrong = dict(w)
        wrong["l0.mlp.correction"] = w["l0.mlp.correction"] * 0
        if 1 < top < n + identity and tokens >= 90:
            assert differs(cfg, wrong, t, taps, 1e-4)
        wrong = dict(w)
        wrong["l0.mlp.shared.sg"] = w["l0.mlp.shared.sg"] * 2
        assert differs(cfg, wrong, t, taps, 1e-4)
        for k in ("expert", "shared"):
            if tokens > 3 and (k == "shared" or n > 2) and cfg["layers"][0]["mlp"][k]["ff"] > 9:
                assert differs(changed(cfg, lambda c: c["layers"][0]["mlp"][k].update(limit=0.3)), w, t, taps, 1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_only_identity_experts_are_chosen(pkg, tmp_path, dtype):
    """No expert has a row: what remains is a multiple of the input beside the shared expert; and the other way round."""
    for sign in (1.0, -1.0):
        cfg, w = experts_only(G.identity_experts(6, 4, 3, 40, 30), 47, False)
        w["l0.mlp.correction"][:] = G.bf16(np.concatenate([-np.ones(6), np.ones(4)]) * sign * 2.0)
        for n in (1, 5, 150, 400):
            agree(pkg, tmp_path / f"{sign}{n}", cfg, w, dtype, n=n)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("block", [0, 16, 32, 64, 128, 256])
def test_experts_of_long_prompts(pkg, tmp_path, forms, knobs, block, dtype):
    """Every block size of the sorted rows, up to the 256-row tiles, with experts that receive few rows or none."""
    knobs.set(MOE_ROWS_BLOCK=block)
    for n, identity, top, tokens in ((4, 2, 2, 400), (9, 1, 3, 110), (6, 6, 1, 75), (12, 3, 2, 500)):
        cfg, w = experts_only(G.identity_experts(n, identity, top, 48, 64), 44, dtype == "bfloat16", width=160)
        agree(pkg, tmp_path / str(n), cfg, w, dtype, n=tokens)


def test_choice_ties_take_the_first_experts(pkg, tmp_path):
    cfg, w = experts_only(G.identity_experts(5, 4, 4, 24, 20), 45, False)
    w["l0.mlp.router"][:] = 0.0
    w["l0.mlp.correction"][:] = 0.0
    agree(pkg, tmp_path, cfg, w, "float32", n=20)


@pytest.mark.parametrize("scale", [1.0, 8.0])
@pytest.mark.parametrize("limit", [0.2, 3.0, 50.0])
@pytest.mark.parametrize("dtype", DTYPES)
def test_limits_of_routed_and_shared_experts(pkg, tmp_path, dtype, limit, scale):
    cfg, w = experts_only(G.identity_experts(3, 1, 2, 30, 44, limit, 2.0 / limit), 49, dtype == "bfloat16")
    for k in w:
        if k.endswith((".gate", ".up")):
            w[k] *= scale
    agree(pkg, tmp_path, cfg, w, dtype, n=40, tol=ALONE[dtype] * (1 if scale == 1.0 else 3))


def test_experts_beside_the_shared_one(pkg, cases, knobs):
    """Small batches run the routed experts on a stream of their own: the same ids as in one stream, eagerly and over many replays of the graph
    with eager work between them."""
    cfg, w, path = cases("far")
    prompts = [toks(cfg, n, 190 + n) for n in (5, 40)]
    runs = []
    for tokens in (0, 64):
        knobs.set(LAYER_OVERLAP_MAX_TOKENS=tokens)
        m = load(pkg, path, "float32", tokens=400, seqs=3, max_len=180)
        nxt, _ = m.unified_forward([(i, p, 0, True) for i, p in enumerate(prompts)])
        out = [nxt[None]]
        for steps in (2, 40, 1, 30):
            out.append(m.decode_steps([0, 1], nxt, steps))
            nxt = out[-1][-1]
            m.unified_forward([(7, toks(cfg, 9, steps), 0, True)])
            m.release(7)
        runs.append(np.concatenate(out))
    assert np.array_equal(*runs)


# ── cache and sizes ───────────────────────────────────────────────────────────────────────────────────────────────────────
@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_are_used_again(pkg, cases, dtype):
    """A pool of six pages, twelve requests one after the other with different lengths: every one must be what it is alone; a request
    too many is refused without side effects."""
    cfg, w, path = cases("far")
    m = load(pkg, path, dtype, tokens=96, seqs=2, blocks=6)
    assert m.state_slots() == (0, 0)
    live = {}
    for i in range(12):
        n = [33, 7, 48, 20][i % 4]
        t = toks(cfg, n, 100 + i)
        if len(live) == 2:
            m.release(live.pop(min(live)))
        assert rel(feed(m, 200 + i, t, [[n], [5, 1], [2]][i % 3]), L.forward(cfg, w, t)) < TOL[dtype], i
        live[i] = 200 + i
    with pytest.raises(RuntimeError):
        m.forward_rows([(999, toks(cfg, 90, 1), 0)], [])
    for s in live.values():
        m.release(s)
    assert m.kv_slot_capacity_snapshot()["free_blocks"] == 6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["far", "talks"])
def test_rows_do_not_depend_on_batch_mates_or_pages(pkg, cases, name, dtype):
    """The same prompt in a fresh pool, in scattered pages, and beside others: equal to rounding, far below the bound to the oracle."""
    cfg, w, path = cases(name)
    t = toks(cfg, 90, 7)
    m = load(pkg, path, dtype, tokens=400, seqs=4)
    alone = feed(m, 1, t, [90])
    m.release(1)
    for s in (2, 3):
        m.forward_rows([(s, toks(cfg, 37, s), 0)], [])
    m.forward_rows([(4, t[:17], 0)], [])
    m.release(2)
    got = [m.forward_rows([(4, t[17:18], 17), (3, toks(cfg, 40, 9), 37)], [0])]
    got.append(m.forward_rows([(5, toks(cfg, 20, 5), 0), (4, t[18:], 18), (3, toks(cfg, 1, 9), 77)], list(range(20, 92))))
    assert rel(np.concatenate(got), alone[17:]) < (3e-6 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_short_and_long_portions_in_one_batch(pkg, cases, dtype):
    """Runs of decoded tokens and short portions between long ones: each takes its own form of attention."""
    cfg, w, path = cases("talks")
    seqs = {i: toks(cfg, n, 500 + i) for i, n in enumerate((60, 70, 40, 33, 90, 25, 64))}
    want = {i: L.forward(cfg, w, t) for i, t in seqs.items()}
    m = load(pkg, path, dtype, tokens=420, seqs=7)
    start = {0: 59, 1: 10, 2: 37, 3: 32, 4: 0, 5: 23, 6: 7}
    m.forward_rows([(i, seqs[i][:n], 0) for i, n in start.items() if n], [])
    items = [(i, seqs[i][start[i]:], start[i]) for i in seqs]
    rows = m.forward_rows(items, list(range(sum(len(x[1]) for x in items))))
    at = 0
    for i, t, n in items:
        assert rel(rows[at:at + len(t)], want[i][n:]) < TOL[dtype], i
        at += len(t)


def test_missing_and_misshapen_weights_are_named(pkg, tmp_path):
    cfg = G.FORORAX["far"]
    w = G.weights(cfg, 1)
    for name, new in (("l0.norm1", None), ("l1.mix.sink", np.zeros(4, np.float32)), ("l1.mlp.e4.down", None), ("l0.mlp.correction", np.zeros(7, np.float32)), ("pos", np.zeros((599, 100), np.float32)),
                      ("l1.mix.talk", np.zeros((6, 5), np.float32)), ("head", None), ("l0.mlp.shared.sg", np.zeros((2, 100), np.float32)), ("l1.mix.g", None), ("l3.mix.o.b", None),
                      ("l0.mix.r2", np.zeros(3, np.float32)), ("l2.mix.q.norm", np.zeros(120, np.float32)), ("l3.mix.v.b", np.zeros(3, np.float32))):
        bad = {k: v for k, v in w.items() if k != name}
        if new is not None:
            bad[name] = new
        with pytest.raises(RuntimeError, match=name.replace(".", r"\.")):
            load(pkg, G.write_checkpoint(tmp_path / name, cfg, bad), "bfloat16")
