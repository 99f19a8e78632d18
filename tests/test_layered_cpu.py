"""Layered architectures without a GPU: config.json → layer descriptions, refusals, and the oracle's own invariants."""
import json

import numpy as np
import pytest

from tests import layered_gen as G
from tests import layered_oracle as L


@pytest.fixture(scope="module")
def pkg():
    import __graft_entry__ as ge
    p = ge.load_package()
    p.load_library()
    return p


def _write(tmp_path, cfg):
    return G.write_checkpoint(tmp_path, cfg, {"embed": np.zeros((2, 2), np.float32)})


@pytest.mark.parametrize("name", list(G.NERENEX))
def test_config_becomes_layer_specs(pkg, tmp_path, name):
    cfg = G.CONFIGS[name]
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    d, arch, tied = ck.model_config(777)
    assert arch == "Nerenex" and tied and (d["hidden"], d["vocab"], d["num_layers"], d["max_seq_len"]) == (cfg["width"], cfg["vocab"], len(cfg["layers"]), 777)
    assert abs(d["rms_eps"] - cfg["norm"]["eps"]) < 1e-9
    lc, specs = ck.layered_config()
    bg = cfg["embedding"]["bigram"]
    assert (lc.bigram_buckets, lc.bigram_mul_prev, lc.bigram_mul_cur) == (bg["buckets"], bg["mul_prev"], bg["mul_cur"])
    assert abs(lc.residual_mult - cfg["residual_mult"]) < 1e-6
    for s, layer in zip(specs, cfg["layers"]):
        m = layer["mixer"]
        assert (s.ff, s.ff_width) == ((1, layer["mlp"]["ff"]) if layer["mlp"] else (0, 0))
        if layer["type"] == "rglru":
            assert (s.mixer, s.rnn_width, s.rnn_blocks, s.conv_taps) == (2, m["width"], m["blocks"], m["conv"])
        else:
            assert (s.mixer, s.heads, s.dim, s.rot_dim, s.vdim, s.q_rank, s.kv_rank, s.rot_dims, s.window) == (
                1, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["rot"]["dims"], m["mask"]["size"])
            assert abs(s.scale - m["scale"]) < 1e-6 and s.rot_base == m["rot"]["base"]


@pytest.mark.parametrize("edit,what", [(lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"), (lambda c: c["layers"][0]["mixer"]["mask"].pop("size"), "size"),
                                       (lambda c: c.pop("residual_mult"), "residual_mult"), (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
                                       (lambda c: c["layers"][1]["mixer"].update(blocks=2.5), "blocks"), (lambda c: c.update(layers=[]), "layers"),
                                       (lambda c: c["norm"].update(eps="x"), "eps")])
def test_incomplete_config_is_refused_by_name(pkg, tmp_path, edit, what):
    cfg = json.loads(json.dumps(G.CONFIGS["odd"]))
    edit(cfg)
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    with pytest.raises(RuntimeError, match=what):
        ck.model_config()
        ck.layered_config()


@pytest.mark.parametrize("edit", [lambda c: c["layers"][0].update(type="convolution"), lambda c: c["layers"][1]["mlp"].update(kind="experts")])
def test_unknown_mechanisms_are_unsupported(pkg, tmp_path, edit):
    from ferrum_infer_rs_amd.backend import Unsupported
    cfg = json.loads(json.dumps(G.CONFIGS["odd"]))
    edit(cfg)
    with pytest.raises(Unsupported):
        pkg.Checkpoint(_write(tmp_path, cfg)).layered_config()


def test_homogeneous_families_are_not_layered(pkg, tmp_path):
    from tests import modelgen
    tm = modelgen.TinyModel(False, layers=2, seed=7)
    modelgen.write_checkpoint(tm, str(tmp_path), "Qwen3ForCausalLM")
    assert pkg.Checkpoint(str(tmp_path)).layered_config() is None


def test_impossible_sizes_are_refused_before_any_device_work(pkg):
    ok = dict(hidden=64, vocab=32, max_seq_len=64, kv_num_blocks=4, max_seqs=1, max_tokens=16)
    lc = pkg.LayeredConfig(dtype=0, residual_mult=1.0)
    for spec in (pkg.LayerSpec(mixer=2, rnn_width=30, rnn_blocks=4, conv_taps=2), pkg.LayerSpec(mixer=1, heads=2, dim=8, rot_dim=4, vdim=8, q_rank=8, kv_rank=8, rot_dims=6, window=4, rot_base=1e4),
                 pkg.LayerSpec(mixer=1, heads=2, dim=8, rot_dim=4, vdim=8, q_rank=8, kv_rank=8, rot_dims=4, window=0, rot_base=1e4), pkg.LayerSpec(mixer=9)):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(lc, [spec]), **ok)


# ── the oracle itself ──
def test_oracle_recurrence_closed_form():
    """Constant inputs: S_t = b (1 − aᵗ) / (1 − a); and the state forgets nothing when the decay is 1."""
    n, lam = 30, np.array([0.3, -2.0])
    u, r, i = np.full((n, 2), 0.7), np.full((n, 2), 0.4), np.full((n, 2), 0.9)
    a = np.exp(-8 * 0.4 * np.log1p(np.exp(lam)))
    t = np.arange(1, n + 1)[:, None]
    want = np.sqrt(1 - a ** 2) * 0.9 * 0.7 * (1 - a ** t) / (1 - a)
    assert np.allclose(L.rglru_scan(u, r, i, lam), want, rtol=1e-12)


def test_oracle_rotation_depends_on_distance_only():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    dot = lambda p, s: float(L.rotate_interleaved(q, [p], 6, 100.0)[0] @ L.rotate_interleaved(k, [s], 6, 100.0)[0])
    assert abs(dot(9, 4) - dot(105, 100)) < 1e-12 and abs(dot(9, 4) - dot(9, 5)) > 1e-3


def test_oracle_activation_is_continuous_with_slope_one_half():
    z = np.array([-1e-6, 1e-6])
    y = L.xielu(z, 0.3, -0.4)
    assert abs((y[1] - y[0]) / 2e-6 - 0.5) < 1e-5 and L.xielu(np.array([-50.0]), 0.3, -0.4)[0] == pytest.approx((0.5 + L.softplus(-0.4)) * 49 - 25)


def test_oracle_window_and_pairs():
    assert L.window_mask(5, 2).sum(axis=1).tolist() == [1, 2, 2, 2, 2]
    assert L.bigram_rows([4, 4, 9], 7, 3, 2).tolist() == [7, (4 * 3 + 4 * 2) % 7, (4 * 3 + 9 * 2) % 7]


# ── Safolorn ──
@pytest.mark.parametrize("name", list(G.SAFOLORN))
def test_safolorn_config_becomes_layer_specs(pkg, tmp_path, name):
    cfg = G.SAFOLORN[name]
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    d, arch, tied = ck.model_config(555)
    assert arch == "Safolorn" and not tied and (d["hidden"], d["vocab"], d["num_layers"], d["max_seq_len"]) == (cfg["width"], cfg["vocab"], len(cfg["layers"]), 555)
    assert abs(d["rms_eps"] - cfg["norm"]["eps"]) < 1e-8
    lc, specs = ck.layered_config()
    assert (lc.block, lc.token_side_dim, lc.untied_head, lc.bigram_buckets) == (1, cfg["token_side"]["dim"], 1, 0)
    for s, layer in zip(specs, cfg["layers"]):
        m, ff = layer["mixer"], layer["mlp"]
        y = m["rot"].get("scaling")
        assert (s.mixer, s.heads, s.dim, s.rot_dim, s.vdim, s.q_rank, s.kv_rank, s.rot_dims, s.window, s.attn_flags) == (
            1, m["heads"], m["dim"], m["rot_dim"], m["vdim"], 0, m["kv_rank"], m["rot"]["dims"], -1, 3)
        assert s.kv_source == m.get("kv_from", -1) + 1 and s.rot_base == m["rot"]["base"] and abs(s.scale - m["scale"]) < 1e-6
        assert (s.rot_factor, s.rot_original, s.rot_fast, s.rot_slow) == ((y["factor"], y["original"], y["fast"], y["slow"]) if y else (0, 0, 0, 0))
        if not ff:
            assert (s.ff, s.ff_width) == (0, 0)
        elif ff["kind"] == "dense":
            assert (s.ff, s.ff_width) == (2, ff["ff"]) and abs(s.ff_limit - ff["limit"]) < 1e-6
        else:
            assert (s.ff, s.ff_width, s.experts, s.top) == (3, ff["expert"]["ff"], ff["router"]["experts"], ff["router"]["top"])


@pytest.mark.parametrize("edit,what", [(lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"), (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
                                       (lambda c: c["layers"][1]["mlp"]["router"].pop("top"), "top"), (lambda c: c["layers"][1]["mlp"].pop("expert"), "expert"),
                                       (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), "slow"), (lambda c: c.pop("token_side"), "token_side"),
                                       (lambda c: c["layers"][0]["mixer"].update(kv_from=0), "kv_from"), (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "kv_from"),
                                       (lambda c: c["layers"][2]["mixer"].pop("scale"), "scale")])
def test_incomplete_safolorn_config_is_refused_by_name(pkg, tmp_path, edit, what):
    cfg = json.loads(json.dumps(G.SAFOLORN["sinks"]))
    edit(cfg)
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    with pytest.raises(RuntimeError, match=what):
        ck.model_config()
        ck.layered_config()


@pytest.mark.parametrize("edit", [lambda c: c["layers"][0].update(type="rglru"), lambda c: c["layers"][1]["mlp"].update(kind="sparse")])
def test_unknown_safolorn_mechanisms_are_unsupported(pkg, tmp_path, edit):
    from ferrum_infer_rs_amd.backend import Unsupported
    cfg = json.loads(json.dumps(G.SAFOLORN["sinks"]))
    edit(cfg)
    with pytest.raises(Unsupported):
        pkg.Checkpoint(_write(tmp_path, cfg)).layered_config()


def test_impossible_parallel_blocks_are_refused_before_any_device_work(pkg):
    ok = dict(hidden=64, vocab=32, max_seq_len=64, kv_num_blocks=4, max_seqs=1, max_tokens=16)
    at = dict(mixer=1, heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=8, rot_dims=4, window=-1, rot_base=1e4, attn_flags=3)
    lc = pkg.LayeredConfig(block=1, token_side_dim=8, untied_head=1, residual_mult=1.0)
    S = pkg.LayerSpec
    for specs in ([S(**at, ff=1, ff_width=8)], [S(**at, ff=2, ff_width=0)], [S(**at, ff=3, ff_width=8, experts=4, top=5)], [S(**at, ff=3, ff_width=8, experts=600, top=2)],
                  [S(mixer=2, rnn_width=32, rnn_blocks=4, conv_taps=2)], [S(**at, kv_source=1)], [S(**at), S(**at, kv_source=1), S(**at, kv_source=2)],
                  [S(**at), S(**{**at, "kv_rank": 16}, kv_source=1)], [S(**at, rot_factor=2.0)]):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(lc, specs), **{**ok, "num_layers": len(specs)})
    for bad in (pkg.LayeredConfig(block=2), pkg.LayeredConfig(block=0, token_side_dim=8)):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(bad, [S(**at)]), **ok)


def test_oracle_sink_and_routing():
    s = np.array([[[1.0, 2.0], [0.5, 0.5]]])
    p = L.softmax_with_sink(s[0], L.window_mask(2, 2), 0.7)
    assert p[0].tolist() == pytest.approx([np.exp(1.0) / (np.exp(1.0) + np.exp(0.7)), 0.0]) and p[1].sum() == pytest.approx(2 * np.exp(0.5) / (2 * np.exp(0.5) + np.exp(0.7)))
    ids, w = L.route(np.array([[0.1, 3.0, 2.0, 3.0]]), 3)
    assert ids[0].tolist() == [1, 3, 2] and w.sum() == pytest.approx(1.0) and w[0, 2] == pytest.approx(np.exp(-1.0) / (2 + np.exp(-1.0)))


def test_oracle_rotation_scaling_keeps_fast_pairs_and_slows_slow_ones():
    f, size = L.yarn(16, 100.0, 8.0, 64, 8.0, 0.5)
    plain = [100.0 ** (-2.0 * i / 16) for i in range(8)]
    assert f[0] == plain[0] and f[-1] == pytest.approx(plain[-1] / 8.0) and all(p / 8.0 <= g <= p for g, p in zip(f, plain)) and size == pytest.approx(1 + 0.1 * np.log(8.0))


# ── Segetar ──
@pytest.mark.parametrize("name", list(G.SEGETAR))
def test_segetar_config_becomes_layer_specs(pkg, tmp_path, name):
    cfg = G.SEGETAR[name]
    w = {f"l{i}.mix.right.a1": np.zeros((3 + i, cfg["width"]), np.float32) for i, l in enumerate(cfg["layers"]) if l["type"] == "parallel"}
    ck = pkg.Checkpoint(G.write_checkpoint(tmp_path, cfg, {"embed": np.zeros((2, 2), np.float32), **w}))
    d, arch, tied = ck.model_config(555)
    assert arch == "Segetar" and not tied and (d["hidden"], d["vocab"], d["num_layers"], d["max_seq_len"]) == (cfg["width"], cfg["vocab"], len(cfg["layers"]), 555)
    assert abs(d["rms_eps"] - cfg["norm"]["eps"]) < 1e-8
    lc, specs = ck.layered_config()
    lp = cfg.get("loop", {"start": 0, "stop": 0, "times": 0})
    assert (lc.block, lc.token_side_dim, lc.untied_head, lc.bigram_buckets, lc.loop_start, lc.loop_stop, lc.loop_times) == (2, 0, 1, 0, lp["start"], lp["stop"], lp["times"])
    for i, (s, layer) in enumerate(zip(specs, cfg["layers"])):
        m, ff = layer["mixer"], layer["mlp"]
        if layer["type"] == "mamba1":
            assert (s.mixer, s.mixer2, s.scan_inner, s.scan_state, s.scan_dt_rank, s.conv_taps) == (6, 0, m["inner"], m["state"], m["dt_rank"], m["conv"])
        else:
            l, r, gated = m["left"], m["right"], layer["type"] == "parallel"
            assert (s.mixer, s.mixer2, s.join, s.attn_flags) == (3, 4 if gated else 5, 0 if gated else 1, 4 if gated else 1)
            assert (s.heads, s.kv_heads, s.dim, s.vdim, s.window) == (l["heads"], l["kv_heads"], l["dim"], l["vdim"], l["mask"]["size"]) and abs(s.scale - l["scale"]) < 1e-6
            assert (s.lin_heads, s.lin_dim, s.lin_vdim) == (r["heads"], r["dim"], r["vdim"])
            if gated:
                assert (s.rot_dims, s.rot_base, s.lin_rot_dims, s.lin_rank) == (l["rot"]["dims"], l["rot"]["base"], 0, 3 + i)
                assert [s.lin_tau, s.left_scale, s.right_scale] == pytest.approx([r["tau"], m["left_scale"], m["right_scale"]])
            else:
                assert (s.rot_dims, s.lin_rot_dims, s.lin_rot_base) == (0, r["rot"]["dims"], r["rot"]["base"])
        if not ff:
            assert (s.ff, s.ff_width) == (0, 0)
        elif ff["kind"] == "dense":
            assert (s.ff, s.ff_width) == (4, ff["ff"])
        else:
            r = ff["router"]
            assert (s.ff, s.ff_width, s.experts, s.top, s.route_groups, s.route_keep) == (5, ff["expert"]["ff"], r["experts"], r["top"], r["groups"]["count"], r["groups"]["keep"])
            assert abs(s.route_scale - r["scale"]) < 1e-6


@pytest.mark.parametrize("edit,what", [(lambda c: c["layers"][0]["mixer"]["left"].pop("kv_heads"), "kv_heads"), (lambda c: c["layers"][0]["mixer"]["left"]["mask"].pop("size"), "size"),
                                       (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5]), "decay"), (lambda c: c["layers"][0]["mixer"]["right"]["decay"].__setitem__(1, 1.5), "decay"),
                                       (lambda c: c["layers"][0]["mlp"]["router"]["groups"].pop("keep"), "keep"), (lambda c: c["layers"][0]["mlp"]["router"].pop("scale"), "scale"),
                                       (lambda c: c["layers"][1]["mixer"].pop("dt_rank"), "dt_rank"), (lambda c: c["layers"][2]["mixer"].pop("left_scale"), "left_scale"),
                                       (lambda c: c["layers"][2]["mixer"]["right"].pop("tau"), "tau"), (lambda c: c["loop"].pop("times"), "times"), (lambda c: c["loop"].update(stop=1), "loop"),
                                       (lambda c: c["layers"][0]["mixer"]["right"]["rot"].pop("base"), "base")])
def test_incomplete_segetar_config_is_refused_by_name(pkg, tmp_path, edit, what):
    cfg = json.loads(json.dumps(G.SEGETAR["loop"]))
    edit(cfg)
    ck = pkg.Checkpoint(G.write_checkpoint(tmp_path, cfg, {"l2.mix.right.a1": np.zeros((5, 100), np.float32)}))
    with pytest.raises(RuntimeError, match=what):
        ck.model_config()
        ck.layered_config()


def test_decay_rank_is_the_shape_of_its_projection(pkg, tmp_path):
    with pytest.raises(RuntimeError, match=r"l2\.mix\.right\.a1"):
        pkg.Checkpoint(_write(tmp_path, G.SEGETAR["loop"])).layered_config()


@pytest.mark.parametrize("edit", [lambda c: c["layers"][0].update(type="rglru"), lambda c: c["layers"][1]["mlp"].update(kind="sparse")])
def test_unknown_segetar_mechanisms_are_unsupported(pkg, tmp_path, edit):
    from ferrum_infer_rs_amd.backend import Unsupported
    cfg = json.loads(json.dumps(G.SEGETAR["loop"]))
    edit(cfg)
    with pytest.raises(Unsupported):
        pkg.Checkpoint(_write(tmp_path, cfg)).layered_config()


def test_impossible_pre_norm_blocks_are_refused_before_any_device_work(pkg):
    ok = dict(hidden=64, vocab=32, max_seq_len=64, kv_num_blocks=4, max_seqs=1, max_tokens=16)
    S = pkg.LayerSpec
    at = dict(mixer=3, heads=4, kv_heads=2, dim=8, vdim=8, rot_dims=4, window=6, rot_base=1e4, scale=0.3)
    lin = dict(mixer2=4, lin_heads=2, lin_dim=8, lin_vdim=8, lin_rank=3, lin_tau=2.0)
    ex = dict(ff=5, ff_width=8, experts=8, top=2, route_groups=4, route_keep=2, route_scale=1.0)
    lc = pkg.LayeredConfig(block=2, untied_head=1, residual_mult=1.0)
    for spec in (S(**{**at, "kv_heads": 3}), S(**{**at, "window": 0}), S(**{**at, "rot_dims": 10}), S(**{**at, "rot_dims": 3}), S(**at, **{**lin, "lin_rank": 0}), S(**at, **{**lin, "lin_vdim": 300}),
                 S(**at, **{**lin, "lin_tau": 0.0}), S(**at, **{**lin, "mixer2": 5, "lin_rot_dims": 9}), S(**at, **{**lin, "mixer2": 2}), S(**at, **lin, join=7), S(mixer=1), S(mixer=2),
                 S(mixer=6, scan_inner=8, scan_state=0, scan_dt_rank=1, conv_taps=2), S(mixer=6, scan_inner=8, scan_state=300, scan_dt_rank=1, conv_taps=2),
                 S(mixer=6, scan_inner=8, scan_state=4, scan_dt_rank=1, conv_taps=2, mixer2=4), S(**at, **{**ex, "route_groups": 3}), S(**at, **{**ex, "route_keep": 5}),
                 S(**at, **{**ex, "top": 5}), S(**at, **{**ex, "experts": 516}), S(**at, ff=1, ff_width=8), S(**at, ff=4, ff_width=0)):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(lc, [spec]), **{**ok, "num_layers": 1})
    for bad in (pkg.LayeredConfig(block=2, untied_head=0), pkg.LayeredConfig(block=2, untied_head=1, bigram_buckets=5), pkg.LayeredConfig(block=2, untied_head=1, loop_times=2, loop_stop=2),
                pkg.LayeredConfig(block=2, untied_head=1, loop_times=2), pkg.LayeredConfig(block=0, loop_times=1, loop_stop=1)):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(bad, [S(**at)]), **{**ok, "num_layers": 1})


@pytest.mark.parametrize("name", list(G.SEGETAR))
def test_segetar_models_choose_experts_by_wide_gaps(monkeypatch, name):
    """What the 16-bit tests of whole models rest on."""
    gaps, route = [], L.grouped_route

    def watch(logits, correction, top, groups, keep, scale):
        choice = (L.sigmoid(logits) + correction).reshape(groups, -1)
        rank = np.sort(choice, axis=1)[:, -2:].sum(axis=1)
        order = np.argsort(-rank, kind="stable")
        inside = -np.sort(-choice[order[:keep]].reshape(-1))
        if keep < groups:
            gaps.append(rank[order[keep - 1]] - rank[order[keep]])
        if top < len(inside):
            gaps.append(inside[top - 1] - inside[top])
        return route(logits, correction, top, groups, keep, scale)
    monkeypatch.setattr(L, "grouped_route", watch)
    cfg = G.SEGETAR[name]
    L.forward(cfg, G.weights(cfg, G.SEEDS[name]), np.random.default_rng(1).integers(0, cfg["vocab"], 120))
    assert min(gaps) > 0.01


def test_oracle_grouped_routing():
    logits = np.log([0.3 / 0.7, 0.9 / 0.1, 0.6 / 0.4, 0.5 / 0.5, 0.95 / 0.05, 0.1 / 0.9])
    ids, w = L.grouped_route(logits, np.zeros(6), 2, 3, 1, 2.0)                # groups 1.2, 1.1, 1.05
    assert ids.tolist() == [1, 0] and w == pytest.approx([2.0 * 0.9 / 1.2, 2.0 * 0.3 / 1.2])
    ids, w = L.grouped_route(logits, np.array([0, -2.0, 0, 0, -3.0, -3.0]), 3, 3, 2, 1.0)
    assert ids.tolist() == [2, 3, 0] and w == pytest.approx(np.array([0.6, 0.5, 0.3]) / 1.4)


def test_oracle_decayed_state_closed_form():
    n = 12
    q, k, v = np.ones((n, 1, 1)), np.ones((n, 1, 1)), np.full((n, 1, 2), 3.0)
    o = L.decayed_state(q, k, v, np.full((n, 1, 1), 0.5))
    assert np.allclose(o[:, 0, 1], 6.0 * (1 - 0.5 ** np.arange(1, n + 1)))


def test_oracle_layer_runs():
    layers = [None] * 4
    assert L.layer_runs({"layers": layers, "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, -1), (1, 0), (2, 0), (1, 1), (2, 1), (3, -1)]
    assert L.layer_runs({"layers": layers}) == [(i, -1) for i in range(4)]


# ── Fororax ──
@pytest.mark.parametrize("name", list(G.FORORAX))
def test_fororax_config_becomes_layer_specs(pkg, tmp_path, name):
    cfg = G.FORORAX[name]
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    d, arch, tied = ck.model_config(555)
    assert arch == "Fororax" and not tied and (d["hidden"], d["vocab"], d["num_layers"], d["max_seq_len"]) == (cfg["width"], cfg["vocab"], len(cfg["layers"]), 555)
    assert ck.model_config(0)[0]["max_seq_len"] == ck.model_config(10 ** 6)[0]["max_seq_len"] == cfg["max_positions"]      # learned positions end there
    lc, specs = ck.layered_config()
    assert (lc.block, lc.untied_head, lc.bigram_buckets, lc.token_side_dim, lc.loop_times, lc.position_rows) == (3, 1, 0, 0, 0, cfg["max_positions"])
    assert [lc.stream_mult, lc.embed_scale, lc.logit_softcap] == pytest.approx([cfg["postln_alpha"], cfg["embedding"]["scale"], cfg["logit_softcap"]])
    for s, layer in zip(specs, cfg["layers"]):
        m, ff = layer["mixer"], layer["mlp"]
        assert (s.mixer, s.mixer2, s.window, s.rot_dims) == (3, 0, -1, 0) and s.attn_flags == (1 | 8 | 16 if layer["type"] == "attention" else 1 | 2 | 4 | 8 | 32 | 64 | 128)
        assert (s.heads, s.kv_heads, s.dim, s.vdim, s.kv_source) == (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m.get("kv_from", -1) + 1) and abs(s.scale - m["scale"]) < 1e-6
        if not ff:
            assert (s.ff, s.ff_width, s.shared_width) == (0, 0, 0)
            continue
        r = ff["router"]
        assert (s.ff, s.ff_width, s.shared_width, s.experts, s.identity_experts, s.top) == (6, ff["expert"]["ff"], ff["shared"]["ff"], r["experts"], r["identity"], r["top"])
        assert [s.ff_limit, s.shared_limit] == pytest.approx([ff["expert"]["limit"], ff["shared"]["limit"]])


@pytest.mark.parametrize("edit,what", [(lambda c: c["layers"][0]["mixer"].pop("kv_heads"), "kv_heads"), (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
                                       (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"), (lambda c: c["layers"][2]["mixer"].update(kv_from=0.5), "kv_from"),
                                       (lambda c: c["layers"][0]["mlp"]["router"].pop("identity"), "identity"), (lambda c: c["layers"][0]["mlp"]["router"].pop("top"), "top"),
                                       (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"), (lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"), "limit"),
                                       (lambda c: c["layers"][0]["mlp"].pop("shared"), "shared"), (lambda c: c.pop("postln_alpha"), "postln_alpha"), (lambda c: c.pop("logit_softcap"), "logit_softcap"),
                                       (lambda c: c["embedding"].pop("scale"), "scale"), (lambda c: c.pop("max_positions"), "max_positions"), (lambda c: c.update(max_positions=0), "max_positions")])
def test_incomplete_fororax_config_is_refused_by_name(pkg, tmp_path, edit, what):
    cfg = json.loads(json.dumps(G.FORORAX["far"]))
    edit(cfg)
    ck = pkg.Checkpoint(_write(tmp_path, cfg))
    with pytest.raises(RuntimeError, match=what):
        ck.model_config()
        ck.layered_config()


@pytest.mark.parametrize("edit", [lambda c: c["layers"][0].update(type="rglru"), lambda c: c["layers"][1]["mlp"].update(kind="dense")])
def test_unknown_fororax_mechanisms_are_unsupported(pkg, tmp_path, edit):
    from ferrum_infer_rs_amd.backend import Unsupported
    cfg = json.loads(json.dumps(G.FORORAX["far"]))
    edit(cfg)
    with pytest.raises(Unsupported):
        pkg.Checkpoint(_write(tmp_path, cfg)).layered_config()


def test_impossible_post_norm_blocks_are_refused_before_any_device_work(pkg):
    ok = dict(hidden=64, vocab=32, max_seq_len=64, kv_num_blocks=4, max_seqs=1, max_tokens=16)
    S = pkg.LayerSpec
    at = dict(mixer=3, heads=4, kv_heads=2, dim=8, vdim=8, window=-1, scale=0.3, attn_flags=9)
    ex = dict(ff=6, ff_width=8, ff_limit=1.0, experts=4, identity_experts=2, top=2, route_groups=1, route_keep=1, route_scale=1.0, shared_width=8, shared_limit=1.0)
    lc = pkg.LayeredConfig(block=3, untied_head=1, residual_mult=1.0, stream_mult=2.0, position_rows=64)
    for specs in ([S(**{**at, "kv_heads": 3})], [S(**at, kv_source=1)], [S(**at), S(**{**at, "dim": 9}, kv_source=1)], [S(**at), S(**{**at, "heads": 6, "kv_heads": 3}, kv_source=1)],
                  [S(**at), S(**at, kv_source=1), S(**at, kv_source=2)], [S(**at), S(**{**at, "attn_flags": 1}, kv_source=1)], [S(**{**at, "attn_flags": 9 | 16 | 32})], [S(**{**at, "attn_flags": 8 | 64})],
                  [S(**at, **{**ex, "top": 7})], [S(**at, **{**ex, "experts": 0})], [S(**at, **{**ex, "identity_experts": -1})], [S(**at, **{**ex, "experts": 510, "identity_experts": 3})],
                  [S(**at, ff=5, ff_width=8, experts=4, top=2, route_groups=1, route_keep=1, route_scale=1.0, shared_width=8)], [S(**at, ff=2, ff_width=8)]):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(lc, specs), **{**ok, "num_layers": len(specs)})
    for bad in (pkg.LayeredConfig(block=3, untied_head=1, position_rows=63), pkg.LayeredConfig(block=3, untied_head=0), pkg.LayeredConfig(block=3, untied_head=1, loop_times=1, loop_stop=1),
                pkg.LayeredConfig(block=3, untied_head=1, logit_softcap=-1.0)):
        with pytest.raises(RuntimeError):
            pkg.HipModel(layered=(bad, [S(**at)]), **{**ok, "num_layers": 1})
    with pytest.raises(RuntimeError, match="identity"):                        # (copies of the input are part of the post-norm sum)
        pkg.HipModel(layered=(pkg.LayeredConfig(block=2, untied_head=1), [S(**at, **ex)]), **{**ok, "num_layers": 1})


@pytest.mark.parametrize("name", list(G.FORORAX))
def test_fororax_models_choose_experts_by_wide_gaps(monkeypatch, name):
    """What the 16-bit tests of whole models rest on."""
    gaps, route = [], L.corrected_softmax_route

    def watch(logits, correction, top):
        e = np.exp(logits - logits.max())
        choice = -np.sort(-(e / e.sum() + correction))
        if top < len(choice):
            gaps.append(choice[top - 1] - choice[top])
        return route(logits, correction, top)
    monkeypatch.setattr(L, "corrected_softmax_route", watch)
    cfg = G.FORORAX[name]
    L.forward(cfg, G.weights(cfg, G.SEEDS[name]), np.random.default_rng(1).integers(0, cfg["vocab"], 120))
    assert min(gaps) > 0.04


def test_oracle_corrected_softmax_routing():
    logits = np.log([0.1, 0.4, 0.3, 0.2])
    ids, w = L.corrected_softmax_route(logits, np.zeros(4), 2)
    assert ids.tolist() == [1, 2] and w == pytest.approx([0.4, 0.3])                       # not over their sum
    ids, w = L.corrected_softmax_route(logits, np.array([0.35, -1.0, 0.0, 0.0]), 2)
    assert ids.tolist() == [0, 2] and w == pytest.approx([0.1, 0.3])


def test_oracle_identity_experts_hand_their_input_on():
    h = np.array([[1.0, -2.0, 3.0]])
    w = {"router": np.zeros((3, 3)), "correction": np.array([-1.0, 0.5, 0.0]), "e0.gate": None}
    assert L.identity_moe(h, w, 1, 2, 1.0)[0] == pytest.approx(2.0 / 3.0 * h[0])


def test_oracle_mixed_heads_and_distances():
    p = np.zeros((2, 1, 2))
    p[0, 0], p[1, 0] = [0.25, 0.75], [1.0, 0.0]
    assert L.mix_heads(p, np.array([[0.0, 2.0], [1.0, -1.0]]))[:, 0].tolist() == [[2.0, 0.0], [-0.75, 0.75]]
    d = L.log_distance(3, 2.0, 0.5)
    assert d[2].tolist() == pytest.approx([2.0 * np.log(2.0), 2.0 * np.log(1.5), 0.0]) and d[0].tolist() == [0.0, 0.0, 0.0]


def test_oracle_softcap_and_head_norm():
    assert L.softcap(np.array([0.01, 1e9, -1e9]), 3.0) == pytest.approx([0.01, 3.0, -3.0], rel=1e-4)
    x = L.head_normed(np.array([[3.0, 4.0, 0.0, 2.0]]), 2, np.array([1.0, 2.0]), 0.0)
    assert x[0].tolist() == [pytest.approx([3 / 12.5 ** 0.5, 8 / 12.5 ** 0.5]), pytest.approx([0.0, 4 / 2 ** 0.5])]
