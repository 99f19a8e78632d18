"""Layered models (Nerenex; for whole models Safolorn, Segetar and Fororax too, see test_safolorn_gpu.py, test_segetar_gpu.py and
test_fororax_gpu.py for their mechanisms) on the device against the plain oracle of tests/layered_oracle.py: every mechanism alone, prompts,
portions and decoding, unequal batches, reuse of pages and slots, window edges with a key that stands out, and greedy generation
through the engine loop.  Models are small and random; none of their numbers come from a checkpoint."""
import json
import os
import subprocess

import numpy as np
import pytest

from tests import layered_gen as G
from tests import layered_oracle as L

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BIN = os.path.join(ROOT, "ferrum-infer-rs_amd", "bin")
# rms over the vocabulary of the difference, relative to the rms of the logits: rounding only
TOL = {"float32": 3e-5, "bfloat16": 4e-2}
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def pkg():
    import torch  # noqa: F401  (ahead of the library: imported later, torch finds no device, and other modules' tests need it)
    import __graft_entry__ as ge
    p = ge.load_package()
    p.load_library()
    return p


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    """name → (config, weights, checkpoint directory)"""
    made = {}

    def get(name):
        if name not in made:
            cfg = G.CONFIGS[name]
            w = G.weights(cfg, G.SEEDS.get(name, 11 + len(made)))
            made[name] = (cfg, w, G.write_checkpoint(tmp_path_factory.mktemp(name), cfg, w))
        return made[name]
    return get


def load(pkg, path, dtype, tokens=512, seqs=4, slots=0, blocks=None, max_len=None):
    return pkg.HipModel.from_checkpoint(path, kv_num_blocks=blocks or (tokens + 15) // 16 + seqs, max_seqs=seqs, max_tokens=max(tokens, seqs),
                                        max_seq_len=max_len or tokens, dtype=dtype, state_slots=slots)


def rel(got, want):
    """Worst row: rms difference over rms of all wanted rows."""
    want = np.asarray(want, np.float64)
    d = np.sqrt(np.mean((np.asarray(got, np.float64) - want) ** 2, axis=-1))
    return float(np.max(d) / np.sqrt(np.mean(want ** 2)))


def feed(m, seq, tokens, cuts):
    """Logits of every token of one sequence fed in portions of the given sizes (the last size repeats)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - at)
        out.append(m.forward_rows([(seq, tokens[at:at + n], at)], list(range(n))))
        at += n
        i += 1
    return np.concatenate(out)


def toks(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.uint32)


# ── each mechanism alone ──────────────────────────────────────────────────────────────────────────────────────────────────
def one_layer(layer, width=72, vocab=50, mult=1.0, **kw):
    return G.config(width, vocab, [layer], mult=mult, **kw)


def taps_of(pkg, tmp_path, cfg, w, dtype, tokens):
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    m.enable_taps()
    m.forward_rows([(1, tokens, 0)], [len(tokens) - 1])
    return m.read_taps(len(tokens))


@pytest.mark.parametrize("dtype", DTYPES)
def test_pair_embedding_across_portions(pkg, tmp_path, dtype):
    """With residual factor 0 the stream stays the embedding: the pair's row for every token, the extra row for the first one, and the
    previous token carried over portion borders, decode steps and a released sequence."""
    cfg = one_layer(G.recurrent(24, 2, 2), mult=0.0, buckets=89, mul_prev=1000003, mul_cur=77)
    w = G.weights(cfg, 3)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    m.enable_taps()
    t = toks(cfg, 23, 5)
    want = L.embed(t, w["embed"].astype(np.float64), w["bigram"].astype(np.float64), 89, 1000003, 77)
    for seq, cuts in ((1, [23]), (2, [1, 2, 7, 1]), (3, [5, 1, 1, 4, 1])):
        at = 0
        while at < len(t):
            n = min(cuts.pop(0) if cuts else 3, len(t) - at)
            m.forward_rows([(seq, t[at:at + n], at)], [])
            assert np.abs(m.read_taps(n)[0] - want[at:at + n]).max() < 1e-6
            at += n
        m.release(seq)


ATTN = [G.attention(3, 20, 6, 36, 44, 52, 9, base=300.0), G.attention(16, 32, 16, 32, 32, 64, 40), G.attention(5, 64, 34, 17, 33, 130, 25, scale=0.3),
        G.attention(1, 5, 2, 3, 4, 7, 2), G.attention(33, 16, 8, 24, 20, 385, 64), G.attention(2, 130, 70, 140, 16, 520, 30)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(ATTN)))
def test_latent_attention_alone(pkg, tmp_path, dtype, i):
    cfg = one_layer(ATTN[i])
    w, t = G.weights(cfg, 20 + i), toks(cfg, 70, 6)
    taps = []
    L.forward(cfg, w, t, taps)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t), taps) < (1e-5 if dtype == "float32" else 3e-2)


REC = [G.recurrent(66, 3, 3), G.recurrent(64, 1, 4), G.recurrent(40, 5, 1), G.recurrent(96, 2, 7)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(REC)))
def test_recurrence_alone(pkg, tmp_path, dtype, i):
    """200 tokens: several scan chunks, decays from near 0 to near 1."""
    cfg = one_layer(REC[i])
    w, t = G.weights(cfg, 30 + i), toks(cfg, 200, 7)
    taps = []
    L.forward(cfg, w, t, taps)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t), taps) < (1e-5 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [41, 160])
def test_feed_forward_alone(pkg, tmp_path, dtype, ff):
    """norm1 = −1 erases the mixer's contribution: what remains is the gated, normed feed-forward with its piecewise activation."""
    cfg = one_layer(G.recurrent(24, 2, 2, ff=ff), mult=0.7)
    w, t = G.weights(cfg, 41), toks(cfg, 33, 8)
    w["l0.norm1"][:] = -1.0
    x = L.embed(t, w["embed"].astype(np.float64), w["bigram"].astype(np.float64), 97, 31, 5)
    f = {k: v.astype(np.float64) for k, v in w.items()}
    want = L.add_sublayer(x, L.dense_ff(x, L.group(f, "l0.mlp.")), f["l0.rg2"], f["l0.rg2.b"], f["l0.norm2"], 0.7, 1e-5)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t)[0], want) < (1e-5 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_gate_and_activation_inputs_stay_finite(pkg, tmp_path, dtype):
    cfg = one_layer(G.recurrent(32, 2, 3, ff=64))
    w, t = G.weights(cfg, 43), toks(cfg, 20, 9)
    for k in ("l0.mlp.up", "l0.rg1", "l0.rg2", "l0.mix.ra", "l0.mix.y"):
        w[k] *= 64.0
    taps = []
    L.forward(cfg, w, t, taps)
    assert rel(taps_of(pkg, tmp_path, cfg, w, dtype, t), taps) < (1e-4 if dtype == "float32" else 0.1)


# ── whole models: prompts, portions, decoding ─────────────────────────────────────────────────────────────────────────────
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_prompt_portions_and_decoding_agree_with_the_oracle(pkg, cases, name, dtype):
    cfg, w, path = cases(name)
    t = toks(cfg, 301, 1)
    want = L.forward(cfg, w, t)
    m = load(pkg, path, dtype)
    errs = {}
    for seq, (label, cuts) in enumerate({"whole": [301], "portions": [2, 3, 64, 17, 65, 2, 129], "twos": [100, 2], "sixteens": [16],
                                         "decode": [240, 1], "from the first token": [1, 1, 1, 1, 1, 33]}.items()):
        errs[label] = rel(feed(m, seq, t, cuts), want)
        m.release(seq)
    assert max(errs.values()) < TOL[dtype], errs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide", "shared", "loop", "talks"])
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5, 6])
def test_first_tokens(pkg, cases, n, name, dtype):
    """Sequences shorter than the convolution, in a slot and blocks that another sequence has just left."""
    cfg, w, path = cases(name)
    m = load(pkg, path, dtype, seqs=1, blocks=10, tokens=160)
    m.forward_rows([(1, toks(cfg, 150, 2), 0)], [])
    m.release(1)
    t = toks(cfg, n, 50 + n)
    assert rel(feed(m, 2, t, [n]), L.forward(cfg, w, t)) < TOL[dtype]
    m.release(2)
    assert rel(feed(m, 3, t, [1]), L.forward(cfg, w, t)) < TOL[dtype]


@pytest.mark.parametrize("tiles", [0, 2])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "wide", "deep", "sinks", "shared", "loop", "all", "far", "talks"])
def test_unequal_batch_against_each_request_alone(pkg, cases, knobs, name, dtype, tiles):
    """Portions of some requests beside single decoded tokens of others, members coming and going; rows against the oracle, and against
    the same rows computed alone to rounding."""
    cfg, w, path = cases(name)
    knobs.set(LATENT_TILES=tiles)
    m = load(pkg, path, dtype, tokens=400, seqs=4)
    seqs = {i: toks(cfg, n, 60 + i) for i, n in enumerate((190, 37, 140, 75))}
    want = {i: L.forward(cfg, w, t) for i, t in seqs.items()}
    plan = [{0: 100, 1: 5}, {0: 1, 1: 1, 2: 70}, {2: 66, 0: 2, 3: 3, 1: 1}, {0: 64, 3: 69, 1: 2}, {0: 1, 2: 1, 3: 1, 1: 1}, {1: 27, 0: 22, 2: 3, 3: 2}]
    at = {i: 0 for i in seqs}
    got = {i: [] for i in seqs}
    for step in plan:
        items = [(i, seqs[i][at[i]:at[i] + n], at[i]) for i, n in step.items()]
        total = sum(step.values())
        rows = m.forward_rows(items, list(range(total)))
        r = 0
        for i, n in step.items():
            got[i].append(rows[r:r + n])
            r += n
            at[i] += n
    alone = load(pkg, path, dtype, tokens=400, seqs=4)
    for i, t in seqs.items():
        g = np.concatenate(got[i])
        assert at[i] == len(t)
        assert rel(g, want[i]) < TOL[dtype]
        assert rel(g, feed(alone, 10 + i, t, [len(t)])) < TOL[dtype]
        alone.release(10 + i)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "loop"])
def test_pages_and_slots_are_used_again(pkg, cases, name, dtype):
    """A pool that holds two short requests, two state slots, twelve requests one after the other with different lengths: every one must
    be what it is alone; exhaustion is refused without side effects."""
    cfg, w, path = cases(name)
    m = load(pkg, path, dtype, tokens=96, seqs=2, slots=2, blocks=6)
    assert m.state_slots() == (2, 2)
    live = {}
    for i in range(12):
        n = [33, 7, 48, 20][i % 4]
        t = toks(cfg, n, 100 + i)
        if len(live) == 2:
            m.release(live.pop(min(live)))
        g = feed(m, 200 + i, t, [[n], [5, 1], [2]][i % 3])
        live[i] = 200 + i
        assert rel(g, L.forward(cfg, w, t)) < TOL[dtype] * (1.5 if (name, dtype) == ("loop", "bfloat16") else 1), i      # (norms of small results, eight layers)
    assert m.state_slots() == (2, 0)
    with pytest.raises(RuntimeError, match="state slots"):
        m.forward_rows([(999, toks(cfg, 3, 1), 0)], [])
    before = m.kv_slot_capacity_snapshot()
    for s in live.values():
        m.release(s)
    assert m.state_slots() == (2, 2) and before["free_blocks"] < 6 and m.kv_slot_capacity_snapshot()["free_blocks"] == 6
    # recurrent state is not kept per block: the prefix cache must never splice such a sequence
    t = toks(cfg, 40, 9)
    feed(m, 500, t, [40])
    m.prefix_cache_register(500, t, 0)
    m.reserve_kv_slots([(501, 40)])
    assert m.prefix_cache_acquire(501, t) == 0


@pytest.mark.parametrize("name", ["deep", "shared", "far"])
def test_prefix_cache_of_an_attention_only_model(pkg, cases, name):
    """Without recurrent layers a cached prefix is spliced in, including the previous token of the pair embedding."""
    cfg, w, path = cases(name)
    m = load(pkg, path, "float32", tokens=160, seqs=2)
    t = toks(cfg, 70, 19)
    feed(m, 1, t[:48], [48])
    m.prefix_cache_register(1, t[:48], 0)
    m.reserve_kv_slots([(2, 70)])
    n = m.prefix_cache_acquire(2, t)
    assert n == 48
    g = m.forward_rows([(2, t[48:], 48)], list(range(22)))
    assert rel(g, L.forward(cfg, w, t)[48:]) < TOL["float32"]


# ── window edges: one key stands out ──────────────────────────────────────────────────────────────────────────────────────
def standout(window, seed=5, kv_rank=64, dim=32, rot=8, vdim=32, heads=4):
    """One attention layer in which token 1's query scores token 0's key far above every other key, wherever they are: the query
    projection of the plain part is α·(direction of token 0's key) ⊗ (token 1's query latent)."""
    cfg = one_layer(G.attention(heads, dim, rot, vdim, 40, kv_rank, window, scale=1.0), width=72, vocab=60)
    w = G.weights(cfg, seed)
    w["bigram"][:] = 0.0
    p = "l0.mix."
    f = {k: v.astype(np.float64) for k, v in w.items()}
    cq = lambda x: L.unit_rms(x @ f[p + "dq"].T, 1e-5) * f[p + "dq.norm"]
    lat = lambda x: L.unit_rms(x @ f[p + "dkv"][:kv_rank].T, 1e-5) * f[p + "dkv.norm"]
    ask, key = cq(f["embed"][1]), lat(f["embed"][0])
    for h in range(heads):
        k = f[p + "uk"][h * dim:(h + 1) * dim] @ key
        uq = np.zeros((dim + rot, 40))
        uq[:dim] = np.outer(k / (k @ k) * 14.0, ask / (ask @ ask))
        w[p + "uq"][h * (dim + rot):(h + 1) * (dim + rot)] = G.bf16(uq)
    return cfg, w


@pytest.mark.parametrize("form,dtype", [("plain", "float32")] + [(f, "bfloat16") for f in ("latent", "pair", "split", "pair split", "expanded", "plain")])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 64, 100])
def test_window_edge(pkg, tmp_path, knobs, forms, window, form, dtype):
    """Token 0 stands exactly on the last visible place, or one further back, for query token 1 — in a prompt, in a portion and decoded,
    with the window's edge at every kind of place within a page.  The oracle with a window one off must be far away."""
    knobs.set(LATENT_PLAIN=int(form == "plain"), LATENT_SPLITS=4 if "split" in form else 1, LATENT_TILES=2 if "pair" in form else 1,
              LATENT_EXPAND_MIN_ROWS=2 if form == "expanded" else 0)
    cfg, w = standout(window)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype)
    forms.reset()
    wrong = json.loads(json.dumps(cfg))
    wrong["layers"][0]["mixer"]["mask"]["size"] = window + 1
    seq = 0
    for at in (0, 3, 15, 16):
        for back in (window - 1, window):
            t = np.full(at + back + 1, 7, np.uint32)
            t[2:] = toks(cfg, max(0, len(t) - 2), 70)[:max(0, len(t) - 2)] % 50 + 5
            t[:2] = t[:2] if len(t) < 2 else 9
            t[at] = 0 if back else 1
            t[at + back] = 1
            want = L.forward(cfg, w, t)[-1:]
            if back == window:                                       # a window one larger would see it
                assert rel(L.forward(wrong, w, t)[-1:], want) > 3 * TOL["bfloat16"]
            whole = feed(m, seq, t, [len(t)])[-1:]
            step = feed(m, seq + 1, t, [max(1, len(t) - 1), 1])[-1:]
            parts = feed(m, seq + 2, t, [max(1, len(t) - 2), 2])[-1:]
            for s in range(3):
                m.release(seq + s)
            seq += 3
            assert max(rel(g, want) for g in (whole, step, parts)) < TOL[dtype], (at, back)
    h = forms.hits()
    if form == "plain":
        assert h.get("latent_attn_plain") and not h.get("latent_attn") and not h.get("latent_attn_expanded")
    elif "split" in form or "pair" in form:
        assert bool(h.get("latent_attn_split")) == ("split" in form) and bool(h.get("latent_attn_pair")) == ("pair" in form)
    elif form == "expanded":
        assert h.get("latent_attn_expanded") or window == 1
    else:
        assert h.get("latent_attn") and not h.get("latent_attn_expanded")


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_among_hundreds_at_page_borders(pkg, tmp_path, dtype):
    """The key that stands out sits 290 tokens back, around a page border, in a prompt, decoded, and seen from a long later portion."""
    cfg, w = standout(600)
    m = load(pkg, G.write_checkpoint(tmp_path, cfg, w), dtype, tokens=512)
    far = json.loads(json.dumps(cfg))
    far["layers"][0]["mixer"]["mask"]["size"] = 250
    for i, at in enumerate((14, 15, 16, 17, 31, 32)):
        t = toks(cfg, at + 291, 80) % 50 + 5
        t[at], t[-1] = 0, 1
        want = L.forward(cfg, w, t)[-1:]
        assert rel(L.forward(far, w, t)[-1:], want) > 3 * TOL["bfloat16"]
        for j, cuts in enumerate(([len(t)], [len(t) - 1, 1], [40, 200, 100], [64, 3])):
            assert rel(feed(m, 10 * i + j, t, cuts)[-1:], want) < TOL[dtype], (at, cuts)
            m.release(10 * i + j)


# ── decoding loop, graph, sampling ────────────────────────────────────────────────────────────────────────────────────────
def near_greedy(cfg, w, prompt, out, slack):
    """Every generated token's oracle logit is within `slack` (relative to the logits' rms) of the best one."""
    full = np.concatenate([prompt, out]).astype(np.uint32)
    lg = L.forward(cfg, w, full[:-1])[len(prompt) - 1:]
    gap = lg.max(axis=1) - lg[np.arange(len(out)), out]
    return float(gap.max() / np.sqrt(np.mean(lg ** 2))) <= slack


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "wide", "sinks", "shared", "loop", "all", "far", "talks"])
def test_long_decoding_through_the_graph(pkg, cases, forms, name, dtype):
    """Three sequences of different lengths decode 150 tokens past their windows in one captured step (several replays with eager
    forwards between them); the same ids as eager single steps, and the oracle's choices up to rounding."""
    cfg, w, path = cases(name)
    m = load(pkg, path, dtype, tokens=3 * 260, seqs=4, max_len=260)
    prompts = [toks(cfg, n, 90 + n) for n in (5, 61, 33)]
    first, _ = m.unified_forward([(i, p, 0, True) for i, p in enumerate(prompts)])
    forms.reset()
    ids, out, nxt = [0, 1, 2], [first[None]], first
    for steps in (1, 60, 2, 40):
        out.append(m.decode_steps(ids, nxt, steps))
        nxt = out[-1][-1]
        # eager work between replays: an unrelated sequence comes and goes
        m.unified_forward([(7, toks(cfg, 9, steps), 0, True)])
        m.release(7)
    gen = np.concatenate(out)
    assert forms.hits().get("graph_replay", 0) >= 100
    # eager, one mixed forward per token, continuing from the state the graph left
    for _ in range(46):
        lens = [m.block_table(i)[1] for i in ids]
        nxt, _ = m.unified_forward([(i, [int(t)], n, True) for i, t, n in zip(ids, nxt, lens)])
        gen = np.concatenate([gen, nxt[None]])
    for i, p in enumerate(prompts):
        assert near_greedy(cfg, w, p, gen[:, i], 2e-4 if dtype == "float32" else 0.25)
    # the whole generation again, eagerly, in another model
    e = load(pkg, path, dtype, tokens=3 * 260, seqs=4, max_len=260)
    nxt, _ = e.unified_forward([(i, p, 0, True) for i, p in enumerate(prompts)])
    again = [nxt]
    for s in range(len(gen) - 1):
        nxt, _ = e.unified_forward([(i, [int(t)], len(p) + s, True) for i, (t, p) in enumerate(zip(nxt, prompts))])
        again.append(nxt)
    if dtype == "float32":
        assert np.array_equal(np.stack(again), gen)


@pytest.mark.parametrize("name", ["tiny", "one", "bare", "lone"])
def test_masked_and_penalised_greedy_choice(pkg, cases, name):
    cfg, w, path = cases(name)
    m = load(pkg, path, "float32")
    t = toks(cfg, 20, 4)
    lg = L.forward(cfg, w, t)[-1]
    best = int(np.argmax(lg))
    mask = np.ones(cfg["vocab"], np.uint8)
    mask[best] = 0
    assert int(m.unified_forward([(1, t, 0, True)], token_mask=mask)[0][0]) == int(np.argmax(np.where(mask, lg, -np.inf)))
    pen = np.where(np.arange(len(lg)) == best, lg / 50.0 if lg[best] > 0 else lg * 50.0, lg)
    assert int(m.unified_forward([(2, t, 0, True)], repetition_penalties=[(50.0, [best])])[0][0]) == int(np.argmax(pen))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "sinks", "loop", "far"])
def test_generation_through_the_engine_loop(cases, name, dtype):
    """The command line: admission bounded by two state slots and a small pool, prompts cut by a 24-token budget beside decoding
    sequences, graph decoding in between; greedy ids against the oracle."""
    cfg, w, path = cases(name)
    prompts = [toks(cfg, n, 300 + n) for n in (30, 3, 57, 12, 1, 41)]
    text = ";".join(",".join(str(int(x)) for x in p) for p in prompts)
    cmd = [os.path.join(BIN, "ferrum_hip_serve"), "--model", path, "--dtype", dtype, "--prompt-ids", text, "--concurrency", "4", "--state-slots", "2",
           "--out-len", "20", "--max-batched-tokens", "24", "--kv-blocks", "9", "--dump-tokens"]
    p = subprocess.run(cmd, capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    lines = p.stdout.strip().splitlines()
    head = json.loads(lines[0])
    assert head["model"] == cfg["architecture"] and head["output_tokens"] == 6 * 20 and head["kv_blocks_free_at_exit"] == head["kv_blocks_total"] == 9
    out = {int(l.split(":")[0].split()[1]): np.array(l.split(":")[1].split(), np.int64) for l in lines[1:]}
    for i, pr in enumerate(prompts):
        assert near_greedy(cfg, w, pr, out[i + 1], 2e-4 if dtype == "float32" else 0.25), i


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide", "shared", "all", "talks"])
def test_trace_replay(cases, tmp_path, name, dtype):
    """bin/trace_run: portions beside decoded tokens, requests that pause, end and make room; logits against the oracle."""
    cfg, w, path = cases(name)
    seqs = {f"q{i}": toks(cfg, n, 400 + n) for i, n in enumerate((150, 20, 90, 64, 33))}
    want = {k: L.forward(cfg, w, t) for k, t in seqs.items()}
    plan = [{"q0": 100, "q1": 2}, {"q1": 17, "q2": 30}, {"q0": 1, "q1": 1, "q2": 2, "q3": 64}, {"q0": 49, "q2": 58, "q4": 31}, {"q4": 2}]
    p = subprocess.Popen([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "384"],
                         stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    at = {k: 0 for k in seqs}
    for s, step in enumerate(plan):
        entries, end, rows = [], [], []
        for k, n in step.items():
            pick = sorted({0, n // 2, n - 1}) if not (s == 1 and k == "q2") else []
            entries.append({"id": k, "tokens": [int(x) for x in seqs[k][at[k]:at[k] + n]], "want": pick})
            rows += [want[k][at[k] + j] for j in pick]
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        p.stdin.write(json.dumps({"step": s, "entries": entries, "end": end}) + "\n")
        p.stdin.flush()
        assert p.stdout.readline().strip() == f"done {s}"
        got = np.fromfile(tmp_path / f"{s}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert got.shape[0] == len(rows) and rel(got, rows) < TOL[dtype]
    p.stdin.close()
    assert p.wait(timeout=30) == 0


@pytest.mark.parametrize("name", ["wide", "shared", "sinks", "loop", "talks"])
def test_few_row_and_tile_projections_agree(pkg, cases, knobs, forms, name):
    """The tile kernel in each of its sizes and the few-row kernel on the same portions."""
    cfg, w, path = cases(name)
    t = toks(cfg, 200, 12)
    want = L.forward(cfg, w, t)
    for big, wide, half, ran in ((1, 10 ** 6, 0, "tiled_gemm_big"), (1, 10 ** 6, 10 ** 6, "tiled_gemm_big"), (1, 1, 0, "tiled_gemm_256"), (10 ** 6, 192, 128, "tiled_gemm")):
        knobs.set(TILED_BIG_MIN_TILES=big, TILED_WIDE_MIN_TILES=wide, TILED_WIDE_MIN_K=0, TILED_HALF_MAX_TILES=half)
        m = load(pkg, path, "bfloat16")
        forms.reset()
        assert rel(feed(m, 1, t, [200]), want) < TOL["bfloat16"]
        h = forms.hits()
        assert h.get(ran) and bool(h.get("tiled_gemm_big")) == (big == 1) and bool(h.get("tiled_gemm_256")) == (wide == 1)


def test_missing_and_misshapen_weights_are_named(pkg, tmp_path):
    cfg = G.CONFIGS["tiny"]
    w = G.weights(cfg, 1)
    for name, new in (("l0.mix.ra", None), ("l1.mix.o", np.zeros((40, 15), np.float32)), ("l2.rg1.b", np.zeros(3, np.float32))):
        bad = {k: v for k, v in w.items() if k != name}
        if new is not None:
            bad[name] = new
        with pytest.raises(RuntimeError, match=name.replace(".", r"\.")):
            load(pkg, G.write_checkpoint(tmp_path / name, cfg, bad), "bfloat16")
