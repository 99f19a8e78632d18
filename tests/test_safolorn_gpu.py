"""Safolorn's mechanisms on the device against the plain oracle of tests/layered_oracle.py: each alone through the taps of small models,
with mistakes planted in the oracle where random weights would hide them; whole models, batches and the engine loop are covered with
the other layered architecture in test_layered_gpu.py."""
import json

import numpy as np
import pytest

from tests import layered_gen as G
from tests import layered_oracle as L
from tests.test_layered_gpu import DTYPES, TOL, cases, feed, load, pkg, rel, taps_of, toks  # noqa: F401  (two are fixtures)

pytestmark = pytest.mark.gpu
ALONE = {"float32": 1e-5, "bfloat16": 2e-2}


def model(layers, width=72, vocab=50, side=12, **kw):
    return G.safolorn(width, vocab, side, layers, **kw)


def changed(cfg, edit):
    c = json.loads(json.dumps(cfg))
    edit(c)
    return c


def f64(w):
    return {k: np.asarray(v, np.float64) for k, v in w.items()}


def agree(pkg, tmp_path, cfg, w, dtype, n=70, tol=None, seed=6):
    t, taps = toks(cfg, n, seed), []
    L.forward(cfg, w, t, taps)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t), taps) < (tol or ALONE[dtype])
    return t, taps


def silence(w, *what):
    """Takes a mixer ("mix.o") or the per-layer token input ("side.norm") of every layer out."""
    for k in w:
        if k.split(".", 1)[-1] in what:
            w[k][:] = 0.0


# ── each mechanism alone ──────────────────────────────────────────────────────────────────────────────────────────────────
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("side,width", [(12, 72), (1, 33), (64, 96), (45, 130)])
def test_token_side_alone(pkg, tmp_path, dtype, side, width):
    """Two layers without mixer and feed-forward: each adds its own part of the side embedding, gated by the stream it is given."""
    cfg = model([G.sink_attention(1, 8, 4, 8, 16)] * 2, width=width, side=side)
    w = G.weights(cfg, 3)
    silence(w, "mix.o")
    t, taps = agree(pkg, tmp_path, cfg, w, dtype, tol=ALONE[dtype])
    f, x = f64(w), L.embed(t, w["embed"].astype(np.float64))
    swapped = L.token_side(x, t, L.group(f, "l0.side."), f["side.embed"][:, side:], 1e-5)      # another layer's part would show
    assert rel(swapped, taps[0]) > 0.1


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("limit,scale", [(0.4, 1.0), (2.0, 4.0), (1.0, 32.0), (100.0, 1.0)])
@pytest.mark.parametrize("ff", [41, 160])
def test_clamped_glu_alone(pkg, tmp_path, dtype, ff, limit, scale):
    cfg = model([G.sink_attention(2, 8, 4, 8, 16, mlp=G.glu(ff, limit))])
    w = G.weights(cfg, 41)
    silence(w, "mix.o", "side.norm")
    for part in ("gate", "up"):
        w[f"l0.mlp.{part}"] *= scale
    _, taps = agree(pkg, tmp_path, cfg, w, dtype, n=33, tol=ALONE[dtype] * (3 if scale > 8 else 1))      # (steep: an input's rounding counts 32 times)
    other = []
    L.forward(changed(cfg, lambda c: c["layers"][0]["mlp"].update(limit=1.5 * limit)), w, toks(cfg, 33, 6), other)
    assert (rel(other, taps) > 3e-3) == (limit < 50)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,top,ff", [(7, 3, 41), (16, 1, 64), (5, 5, 20), (1, 1, 33), (70, 6, 24), (130, 2, 40), (300, 7, 9)])
@pytest.mark.parametrize("tokens", [1, 3, 90, 150])
def test_experts_alone(pkg, tmp_path, forms, dtype, n, top, ff, tokens):
    """Routing and sorting in one launch and in two, on every number of experts per lane; 32-bit: routers that read everything."""
    cfg = model([G.sink_attention(2, 8, 4, 8, 16, mlp=G.experts(n, top, ff))])
    w = G.weights(cfg, 43, clear_routes=dtype == "bfloat16")
    silence(w, "mix.o", "side.norm")
    _, taps = agree(pkg, tmp_path, cfg, w, dtype, n=tokens)
    assert bool(forms.hits().get("moe_route_sort")) == (tokens * top <= 1024)
    if top < n and dtype == "float32":                                        # (clear routes leave the last choice little weight)
        other = []
        L.forward(changed(cfg, lambda c: c["layers"][0]["mlp"]["router"].update(top=top + 1)), w, toks(cfg, tokens, 6), other)
        assert rel(other, taps) > 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("block", [0, 16, 32, 64, 128, 256])
def test_experts_of_long_prompts(pkg, tmp_path, forms, knobs, block, dtype):
    """Every block size of the sorted rows, up to the 256-row tiles, with experts that receive few rows or none; an odd number of K steps."""
    knobs.set(MOE_ROWS_BLOCK=block)
    for n, top, tokens in ((4, 2, 400), (9, 3, 110), (6, 1, 75), (12, 2, 500)):
        cfg = model([G.sink_attention(2, 8, 4, 8, 16, mlp=G.experts(n, top, 48))], width=160)
        w = G.weights(cfg, 44)
        silence(w, "mix.o", "side.norm")
        agree(pkg, tmp_path / str(n), cfg, w, dtype, n=tokens)
    h = forms.hits()
    assert bool(h.get("tiled_gemm_grouped_big")) == (dtype == "bfloat16" and (block == 0 or block > 64))
    assert bool(h.get("tiled_gemm_grouped")) == (dtype == "float32" or block <= 64)


def test_experts_beside_the_mixer(pkg, cases, knobs):
    """Small batches run the experts on a stream of their own: the same ids as in one stream, eagerly and over many replays of the graph
    with eager work between them."""
    cfg, w, path = cases("sinks")
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
        for _ in range(20):
            nxt, _ = m.unified_forward([(i, [int(t)], m.block_table(i)[1], True) for i, t in enumerate(nxt)])
            out.append(nxt[None])
        runs.append(np.concatenate(out))
    assert np.array_equal(*runs)


def test_equal_router_logits_take_the_first_experts(pkg, tmp_path):
    cfg = model([G.sink_attention(2, 8, 4, 8, 16, mlp=G.experts(9, 4, 24))])
    w = G.weights(cfg, 45)
    w["l0.mlp.router"][:] = 0.0
    w["l0.mlp.router.b"][:] = 0.0
    agree(pkg, tmp_path, cfg, w, "float32", n=20)


ATTN = [G.sink_attention(3, 20, 6, 36, 52, 300.0, (4.0, 30, 5.0, 1.0)), G.sink_attention(16, 32, 16, 32, 64), G.sink_attention(5, 64, 34, 17, 130, 1e4, (1.5, 50, 8.0, 2.0), scale=0.3),
        G.sink_attention(1, 5, 2, 3, 7, yarn=(8.0, 20, 3.0, 2.9)), G.sink_attention(33, 16, 8, 24, 385, 50.0, (2.0, 4096, 32.0, 1.0)), G.sink_attention(2, 130, 70, 140, 520)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(ATTN)))
def test_attention_alone(pkg, tmp_path, dtype, i):
    cfg = model([ATTN[i]])
    w = G.weights(cfg, 20 + i)
    silence(w, "side.norm")
    w["l0.mix.o"] *= 4.0
    t, taps = agree(pkg, tmp_path, cfg, w, dtype, tol=ALONE[dtype] * (1 if dtype == "float32" else 2))
    wrong = dict(w)
    wrong["l0.mix.sink"] = w["l0.mix.sink"] * cfg["layers"][0]["mixer"]["scale"]                # the sink is not a scaled score
    other = []
    L.forward(cfg, wrong, t, other)
    assert rel(other, taps) > 3 * ALONE["float32"]


@pytest.mark.parametrize("yarn", [(4.0, 30, 5.0, 1.0), (3.0, 200, 400.0, 300.0), (2.0, 10, 0.5, 0.1), (1.0, 64, 4.0, 1.0), (16.0, 64, 2.0, 2.0)])
def test_scaled_rotation(pkg, tmp_path, yarn):
    """All pairs slowed, none, some on the ramp, ramp of no width; the plain part of queries and keys is zero, so positions are all there is."""
    cfg = model([G.sink_attention(2, 8, 16, 24, 16, 100.0, yarn, scale=1.0)])
    w = G.weights(cfg, 51)
    silence(w, "side.norm")
    w["l0.mix.uk"][:] = 0.0
    w["l0.mix.o"] *= 2.0
    t, taps = agree(pkg, tmp_path, cfg, w, "float32", n=120)
    other = []
    L.forward(changed(cfg, lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling")), w, t, other)
    assert (rel(other, taps) > 1e-3) == (yarn[0] != 1.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[70], [1], [40, 3, 2, 1], [20, 50]])
def test_latents_of_an_earlier_layer(pkg, tmp_path, dtype, cuts):
    """Layers 2 and 3 read what layers 0 and 1 have cached, in this portion and in earlier ones, with their own projections."""
    own = [G.sink_attention(4, 16, 8, 16, 32), G.sink_attention(3, 24, 8, 12, 40, 100.0)]
    cfg = model(own + [G.sink_attention(5, 20, 8, 28, 40, 100.0, kv_from=1), G.sink_attention(2, 16, 8, 16, 32, kv_from=0)])
    w, t = G.weights(cfg, 53), toks(cfg, 70, 6)
    w["l2.mix.o"] *= 4.0
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    want = L.forward(cfg, w, t)
    assert rel(feed(m, 1, t, cuts), want) < TOL[dtype]
    plain = changed(cfg, lambda c: [l["mixer"].update(kv_from=0, kv_rank=32, rot={"base": 10000.0, "dims": 8}) for l in c["layers"][2:3]])
    pw = dict(w)
    pw["l2.mix.uk"], pw["l2.mix.uv"] = w["l2.mix.uk"][:, :32], w["l2.mix.uv"][:, :32]
    assert rel(L.forward(plain, pw, t), want) > 3 * TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("eps", [1e-5, 0.3])
def test_norms_with_one_number(pkg, tmp_path, dtype, eps):
    """Gains that differ between the two sublayers and the end; a large epsilon shows where it stands."""
    cfg = model([G.sink_attention(2, 16, 8, 16, 32, mlp=G.glu(50, 1.0)), G.sink_attention(2, 16, 8, 16, 32, mlp=G.experts(6, 2, 30))], eps=eps)
    w = G.weights(cfg, 55)
    w["embed"] *= 0.25
    for k, g in (("l0.norm1", 0.5), ("l0.norm2", 2.0), ("l1.norm1", 1.75), ("l1.norm2", 0.75), ("final.norm", -1.5)):
        w[k] = np.float32(g)
    m, t = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype), toks(cfg, 40, 6)
    assert rel(feed(m, 1, t, [40]), L.forward(cfg, w, t)) < TOL[dtype]


# ── one key stands out ────────────────────────────────────────────────────────────────────────────────────────────────────
def standout(seed=5, kv_rank=64, dim=32, rot=8, vdim=32, heads=4, sink=4.0, score=16.0):
    """One attention layer in which token 1's query scores token 0's key far above every other key and the sink, wherever they are."""
    cfg = model([G.sink_attention(heads, dim, rot, vdim, kv_rank, scale=1.0)], width=72, vocab=60)
    w = G.weights(cfg, seed, clear_routes=False)
    silence(w, "side.norm")
    p, f = "l0.mix.", f64(w)
    h = lambda t: L.unit_rms(f["embed"][t], 1e-5) * f["l0.norm1"]
    ask, key = h(1), L.unit_rms(f[p + "dkv"][:kv_rank] @ h(0), 1e-5) * f[p + "dkv.norm"]
    for a in range(heads):
        k = f[p + "uk"][a * dim:(a + 1) * dim] @ key
        q = np.zeros((dim + rot, 72))
        q[:dim] = np.outer(k / (k @ k) * score, ask / (ask @ ask))
        w[p + "q"][a * (dim + rot):(a + 1) * (dim + rot)] = G.bf16(q)
    w[p + "sink"][:] = sink
    w[p + "o"] *= 2.0
    return cfg, w


FORMS = [("plain", "float32")] + [(f, "bfloat16") for f in ("latent", "pair", "split", "pair split", "expanded", "plain")]


def set_form(knobs, form):
    knobs.set(LATENT_PLAIN=int(form == "plain"), LATENT_SPLITS=4 if "split" in form else 1, LATENT_TILES=2 if "pair" in form else 1,
              LATENT_EXPAND_MIN_ROWS=2 if form == "expanded" else 0)


@pytest.mark.parametrize("form,dtype", FORMS)
def test_far_key_and_future_key(pkg, tmp_path, knobs, forms, form, dtype):
    """The key that stands out sits hundreds of tokens back, at a page border, in a prompt, a portion of two and decoded; standing right
    behind the query it must not be seen."""
    set_form(knobs, form)
    cfg, w = standout()
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
    h = forms.hits()
    assert h.get({"plain": "latent_attn_plain", "expanded": "latent_attn_expanded"}.get(form, "latent_attn" if "split" not in form else "latent_attn_split"))


@pytest.mark.parametrize("form,dtype", FORMS)
@pytest.mark.parametrize("sink", [-60.0, 0.0, 16.0, 90.0])
def test_sink_against_scores(pkg, tmp_path, knobs, form, dtype, sink):
    """A sink far below, among, level with the best score, and far above every score (the heads then add nothing)."""
    set_form(knobs, form)
    cfg, w = standout(sink=sink)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=256)
    t = toks(cfg, 190, 81) % 50 + 5
    t[3], t[189], t[70] = 0, 1, 1
    want = L.forward(cfg, w, t)
    without = dict(w)
    without["l0.mix.sink"] = np.full(4, -1e9, np.float32)
    assert (rel(L.forward(cfg, without, t)[-1:], want[-1:]) > 3 * TOL["bfloat16"]) == (sink > 10)
    for i, cuts in enumerate(([190], [188, 1], [100, 64, 2], [1, 1, 1, 187])):
        assert rel(feed(m, i, t, cuts), want) < TOL[dtype], cuts
        m.release(i)


# ── cache and sizes ───────────────────────────────────────────────────────────────────────────────────────────────────────
@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_are_used_again(pkg, cases, dtype):
    """A pool of six pages, twelve requests one after the other with different lengths: every one must be what it is alone; a request
    too many is refused without side effects; no state slots are asked for."""
    cfg, w, path = cases("sinks")
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
def test_rows_do_not_depend_on_batch_mates_or_pages(pkg, cases, dtype):
    """The same prompt in a fresh pool, in scattered pages, and beside others: equal to rounding, far below the bound to the oracle."""
    cfg, w, path = cases("shared")
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
    assert rel(np.concatenate(got), alone[17:]) < (2e-6 if dtype == "float32" else 2e-2)


def test_missing_and_misshapen_weights_are_named(pkg, tmp_path):
    cfg = G.SAFOLORN["sinks"]
    w = G.weights(cfg, 1)
    for name, new in (("l0.norm1", None), ("l0.mix.sink", np.zeros(4, np.float32)), ("l1.mlp.e6.down", None), ("l1.mlp.router.b", np.zeros(6, np.float32)),
                      ("side.embed", np.zeros((131, 39), np.float32)), ("l2.mix.uk", None), ("head", None), ("l0.mlp.down", np.zeros((100, 74), np.float32))):
        bad = {k: v for k, v in w.items() if k != name}
        if new is not None:
            bad[name] = new
        with pytest.raises(RuntimeError, match=name.replace(".", r"\.")):
            load(pkg, G.write_checkpoint(tmp_path / name, cfg, bad), "bfloat16")
