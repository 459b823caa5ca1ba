"""The plain restatement of Pinepel held against closed forms, the tests' own needles, and the parts of the loader that need
no device."""
import json
import os

import numpy as np

import plan_util as u
from oracle import pinepel_ref as ref

NARROW = dict(heads=9, dim=32, rot=32, vdim=32, kv_rank=64, q_rank=72)
BF16_LIMIT = 0.06  # of the GPU tests


def test_window_off_by_one_would_show():
    """the same needle against an oracle whose window is one token off (planted there): far above every limit used here"""
    cfg = u.config([u.latent(window=50, scale=0.3, **NARROW)], width=96)
    w = u.oracle_weights(u.needle_weights(cfg, 3, key_token=7))
    t = np.random.default_rng(0).integers(8, cfg["vocab"], 160)
    t[64] = 7
    good = ref.forward(cfg, w, t)
    off = json.loads(json.dumps(cfg))
    off["layers"][0]["mixer"]["mask"]["size"] = 51
    bad = ref.forward(off, w, t)
    err = u.rel_rms(bad, good)
    assert err[64 + 50] > 5 * BF16_LIMIT and err[64 + 49] < 1e-9


def test_rotation_keeps_relative_positions():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((1, 1, 12)), rng.standard_normal((1, 1, 12))
    for interleaved in (True, False):
        at = lambda x, p: ref.rotate(x, 500.0, 8, interleaved, start=p)[0, 0]
        np.testing.assert_allclose(at(q, 11) @ at(k, 4), at(q, 107) @ at(k, 100), rtol=1e-10)
        np.testing.assert_array_equal(at(q, 5)[8:], q[0, 0, 8:])
    # the two layouts pair different dimensions: equal after the reordering that maps one on the other
    order = np.r_[np.arange(0, 8, 2), np.arange(1, 8, 2), np.arange(8, 12)]
    np.testing.assert_allclose(ref.rotate(q, 500.0, 8, True, 3)[0, 0][order], ref.rotate(q[..., order], 500.0, 8, False, 3)[0, 0])


def test_delta_rule_without_decay_overwrites():
    """no decay, full steps, one key: the state returns the value written last; an orthogonal key reads nothing"""
    k = np.tile(np.array([1.0, 0.0]), (3, 1, 1))
    v = np.arange(6.0).reshape(3, 1, 2)
    q = np.stack([k[0], k[1], np.array([[0.0, 1.0]])])
    out = ref.delta_rule(q, k, v, np.ones((3, 1, 2)), np.ones((3, 1)))
    np.testing.assert_allclose(out[0], v[0])
    np.testing.assert_allclose(out[1], v[1])
    np.testing.assert_allclose(out[2], 0.0)
    # a decay acts on its own key channel only, before the write
    out = ref.delta_rule(k, k, v, np.array([0.5, 1.0]).reshape(1, 1, 2).repeat(3, 0), np.zeros((3, 1)) + 0.5)
    s = 0.0
    for t in range(3):
        s = 0.5 * s
        s = s + 0.5 * (v[t, 0] - s)
        np.testing.assert_allclose(out[t, 0], s)


def test_short_convolution_and_windows():
    x = np.arange(1.0, 6.0)[:, None]
    np.testing.assert_allclose(ref.short_conv(x, np.array([[100.0, 10.0, 1.0]]))[:, 0], [1, 12, 123, 234, 345])
    np.testing.assert_array_equal(ref.visible(5, 2).sum(1), [1, 2, 2, 2, 2])
    np.testing.assert_array_equal(ref.visible(5, 0).sum(1), [1, 2, 3, 4, 5])
    p = ref.softmax_with_sink(np.zeros((1, 3)), np.log(5.0) * np.ones((1, 1)))
    np.testing.assert_allclose(p, 1 / 8)


def test_loop_order():
    cfg = dict(layers=[None] * 5, loop=dict(start=1, stop=3, times=3))
    assert ref.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    assert ref.layer_runs(dict(layers=[None] * 2, loop=None)) == [(0, False), (1, False)]


def test_directory_is_recognised_by_its_config(tmp_path):
    from xfastertransformer_amd import automodel
    is_plan = lambda p: automodel._lib.xft_automodel_is_plan(os.fsencode(str(p)))
    assert not is_plan(tmp_path)
    (tmp_path / "config.json").write_text("{ not json")
    assert not is_plan(tmp_path)
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "SomethingElse"}))
    assert not is_plan(tmp_path)
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Pinepel", "a": [1, -2.5e3, True, None, "\u00e9\"\\"]}))
    assert is_plan(tmp_path)
    (tmp_path / "config.ini").write_text("[llama]\n")
    assert not is_plan(tmp_path)
