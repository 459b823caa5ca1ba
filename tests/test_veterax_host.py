"""The plain restatement of Veterax held against closed forms; what the GPU tests' inputs would show, with mistakes planted in the
restatement; and the parts of the loader that need no device."""
import json
import math
import os

import numpy as np
import pytest

import veterax_util as u
from oracle import veterax_ref as ref

BF16_LIMIT = 0.06  # of the GPU tests


def test_squashing_norm():
    w = {"n": np.array([2.0, 1.0]), "n.b": np.array([0.5, -1.0]), "n.alpha": np.array(0.5)}
    np.testing.assert_allclose(ref.dynamic_tanh(np.array([[0.0, 1e9], [2.0, -2.0]]), w, "n"),
                               [[0.5, 0.0], [2 * math.tanh(1) + 0.5, -math.tanh(1) - 1]])


def test_rotation():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((1, 1, 14)), rng.standard_normal((1, 1, 14))
    for scaling in (None, dict(factor=8.0, original=40, fast=3.0, slow=0.5)):
        rot = dict(base=300.0, dims=10, scaling=scaling)
        at = lambda x, p: ref.rotate(x, rot, p)[0, 0]
        np.testing.assert_allclose(at(q, 11) @ at(k, 4), at(q, 107) @ at(k, 100), rtol=1e-10)  # only the distance counts
        np.testing.assert_array_equal(at(q, 5)[10:], q[0, 0, 10:])
        grown = np.linalg.norm(at(q, 5)[:10]) / np.linalg.norm(q[0, 0, :10])
        np.testing.assert_allclose(grown, 0.1 * math.log(8.0) + 1.0 if scaling else 1.0)
    # neighbours form a pair: the fastest one turns by one radian a position
    np.testing.assert_allclose(ref.rotate(np.array([[[1.0, 0.0]]]), dict(base=10.0, dims=2), 3)[0, 0], [math.cos(3), math.sin(3)])


def test_context_extension():
    dims, base = 64, 1e4
    plain, _ = ref.yarn(dims, base, None)
    f, mul = ref.yarn(dims, base, dict(factor=4.0, original=1024, fast=16.0, slow=1.0))
    turns = 1024 * plain / (2 * math.pi)
    ratio = f / plain
    assert mul == pytest.approx(1.0 + 0.1 * math.log(4.0))
    np.testing.assert_allclose(ratio[turns > 20], 1.0)
    np.testing.assert_allclose(ratio[turns < 0.8], 0.25)
    assert np.all(np.diff(ratio) <= 1e-12) and ((ratio > 0.3) & (ratio < 0.95)).any()
    # both bounds on one pair: a step, not a division by nothing
    g, _ = ref.yarn(4, 10.0, dict(factor=2.0, original=6.3, fast=1.0, slow=1.0))
    assert np.isfinite(g).all()


def test_softmax_with_sink_and_groups():
    z = np.zeros((3, 4, 2))
    v = np.arange(6.0).reshape(3, 2, 1)
    out = ref.attend(z, np.zeros((3, 2, 2)), v, 1.0, np.log(np.array([1.0, 3.0, 1.0, 1e-30])))
    np.testing.assert_allclose(out[2, :, 0], [(0 + 2 + 4) / 4, (0 + 2 + 4) / 6, (1 + 3 + 5) / 4, (1 + 3 + 5) / 3])
    np.testing.assert_allclose(out[0, :, 0], [0, 0, 0.5, 1.0])
    np.testing.assert_allclose(ref.attend(z, np.zeros((3, 2, 2)), v, 1.0, np.full(4, -99.0), window=2)[2, 3, 0], 4.0)


def test_routing():
    w = {"router": np.eye(4), "correction": np.array([0.0, 0.0, 0.0, 0.9])}
    h = np.log(np.array([[0.1, 0.2, 0.3, 0.4], [0.7, 0.1, 0.15, 0.05]]))
    # the correction chooses, the score weighs, nothing is renormalised
    np.testing.assert_allclose(ref.route(h, w, "", 2), [[0, 0, 0.3, 0.4], [0.7, 0, 0, 0.05]], atol=1e-12)


def test_identity_experts_hand_their_input_through():
    cfg = u.config([(u.attention(), u.moe(experts=1, identity=3, top=1, shared_ff=0))])
    w = u.oracle_weights(u.weights(cfg, 1))
    w["l0.mlp.correction"][:] = [-9, 9, 0, 0]
    h = np.random.default_rng(1).standard_normal((5, cfg["width"]))
    s = ref.softmax(h @ w["l0.mlp.router"].T)
    np.testing.assert_allclose(ref.experts(h, w, "l0.mlp.", cfg["layers"][0]["mlp"]), s[:, 1:2] * h)


def test_steady_routing_is_what_it_says():
    cfg = u.config([(u.attention(), u.moe()), (u.attention(), u.moe(experts=9, identity=1, top=4, shared_ff=0))])
    w = u.oracle_weights(u.steady_weights(cfg, 3))
    t = np.random.default_rng(1).integers(0, cfg["vocab"], 60)
    chosen = []
    full, route = ref.forward(cfg, w, t), ref.route
    try:
        ref.route = lambda h, w_, p, top: chosen.append(route(h, w_, p, top) > 0) or route(h + np.random.default_rng(0).standard_normal(h.shape) * 0.01, w_, p, top)
        shaken = ref.forward(cfg, w, t)
    finally:
        ref.route = route
    assert all(len({tuple(r) for r in c}) > 3 for c in chosen), "the choices do not depend on the token"
    assert u.rel_rms(shaken, full).max() < BF16_LIMIT


# ---- mistakes planted in the restatement show in the outputs the GPU tests look at ----------------------------------------
def planted():
    def other_pairs(x, rot, start=0):
        n = rot["dims"]
        order = np.r_[np.arange(0, n, 2), np.arange(1, n, 2), np.arange(n, x.shape[-1])]
        y = good["rotate"](x[..., np.argsort(order)], rot, start)
        return y[..., order]

    def weights_with_correction(h, w, p, top):
        s = good["route"](h, w, p, top)
        return np.where(s > 0, s + w[p + "correction"], 0.0)

    def renormalised(h, w, p, top):
        s = good["route"](h, w, p, top)
        return s / s.sum(-1, keepdims=True)

    good = {n: getattr(ref, n) for n in ("rotate", "yarn", "attend", "attention", "route", "clamped_glu", "experts", "token_side", "gelu_tanh", "dynamic_tanh")}
    g = good
    return {
        "rotation pairs halves": dict(rotate=other_pairs),
        "no growth of cos and sin": dict(yarn=lambda *a: (g["yarn"](*a)[0], 1.0)),
        "no context extension": dict(yarn=lambda d, b, s: (g["yarn"](d, b, None)[0], g["yarn"](d, b, s)[1])),
        "no sink": dict(attend=lambda q, k, v, s, sink, *a: g["attend"](q, k, v, s, sink - 99, *a)),
        "scaled sink": dict(attend=lambda q, k, v, s, sink, *a: g["attend"](q, k, v, s, sink * s, *a)),
        "values not mixed": dict(attention=lambda h, w, p, m, eps, first: g["attention"](h, w, p, m, eps, None)),
        "correction in the weights": dict(route=weights_with_correction),
        "weights renormalised": dict(route=renormalised),
        "correction ignored": dict(route=lambda h, w, p, top: g["route"](h, dict(w, **{p + "correction": 0 * w[p + "correction"]}), p, top)),
        "no limit": dict(clamped_glu=lambda h, w, p, limit: g["clamped_glu"](h, w, p, 1e9)),
        "identity experts silent": dict(experts=lambda h, w, p, f: g["experts"](h, dict(w), p, f) - g["route"](h, w, p, f["router"]["top"])[:, f["router"]["experts"]:].sum(-1, keepdims=True) * h),
        "no shared expert": dict(experts=lambda h, w, p, f: g["experts"](h, w, p, {k: v for k, v in f.items() if k != "shared"})),
        "side gate without its gelu": dict(gelu_tanh=lambda z: z),
        "side norm missing": dict(token_side=lambda x, w, p, t, eps: (g["gelu_tanh"](x @ w[p + "side.gate"].T) * t) @ w[p + "side.proj"].T * w[p + "side.norm"]),
        "norm without its shift": dict(dynamic_tanh=lambda x, w, p: g["dynamic_tanh"](x, w, p) - w[p + ".b"]),
    }


@pytest.mark.parametrize("name", sorted(planted()))
def test_planted_mistakes_would_show(name):
    cfg = u.config([(u.attention(), u.moe()), (u.attention(), u.moe()), (u.attention(), None)])
    for make in (u.weights, u.steady_weights):
        w = u.oracle_weights(make(cfg, 6))
        t = np.random.default_rng(2).integers(0, cfg["vocab"], 75)
        want = ref.forward(cfg, w, t)
        changes = planted()[name]
        saved = {n: getattr(ref, n) for n in changes}
        try:
            for n, f in changes.items():
                setattr(ref, n, f)
            bad = ref.forward(cfg, w, t)
        finally:
            for n, f in saved.items():
                setattr(ref, n, f)
        err = u.rel_rms(bad, want).max()
        assert err > 1.2 * BF16_LIMIT, (name, make.__name__, err)


def test_needle_decides():
    for dims in (12, 20):
        cfg = u.config([(u.attention(rot=dims, base=5e4, scaling=None), None)], side=0)
        w = u.oracle_weights(u.needle_weights(cfg, 3, key_token=7))
        t = np.random.default_rng(0).integers(8, cfg["vocab"], 200)
        t[64] = 7
        blind = t.copy()
        blind[64] = 9
        assert u.rel_rms(ref.forward(cfg, w, t), ref.forward(cfg, w, blind))[65:].min() > 3 * BF16_LIMIT


def test_directory_is_recognised_by_its_config(tmp_path):
    from xfastertransformer_amd import automodel
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Veterax"}))
    assert automodel._lib.xft_automodel_is_plan(os.fsencode(str(tmp_path)))
