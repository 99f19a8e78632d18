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


@pytest.mark.parametrize("name", list(G.CONFIGS))
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
