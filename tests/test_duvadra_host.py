"""The plain restatement of Duvadra held against closed forms; what the GPU tests' inputs would show, with mistakes planted in the
restatement; and the parts of the loader that need no device."""
import json
import math
import os

import numpy as np
import pytest

import duvadra_util as u
from oracle import duvadra_ref as ref

BF16_LIMIT = 0.06  # of the GPU tests


def test_pair_rows():
    b = dict(buckets=10, mul_prev=3, mul_cur=7)
    np.testing.assert_array_equal(ref.bigram_rows([4, 9, 9, 0], b), [10, (12 + 63) % 10, (27 + 63) % 10, 27 % 10])
    w = dict(embed=np.arange(12.0).reshape(12, 1), bigram=100.0 * np.arange(11.0).reshape(11, 1))
    np.testing.assert_allclose(ref.embed([4, 9], w, dict(scale=0.5, bigram=b))[:, 0], [2.0 + 1000.0, 4.5 + 500.0])


def test_rotation():
    rng = np.random.default_rng(0)
    rot = dict(base=300.0, dims=10)
    q, k = rng.standard_normal(14), rng.standard_normal(14)
    at = lambda x, p: ref.rotate(np.tile(x, (p + 1, 1, 1)), rot)[p, 0]
    np.testing.assert_allclose(at(q, 11) @ at(k, 4), at(q, 107) @ at(k, 100), rtol=1e-10)  # only the distance counts
    np.testing.assert_array_equal(at(q, 5)[10:], q[10:])
    np.testing.assert_allclose(ref.rotate(np.tile([[[1.0, 0.0]]], (4, 1, 1)), dict(base=10.0, dims=2))[3, 0], [math.cos(3), math.sin(3)])


def test_masks():
    np.testing.assert_array_equal(ref.window_mask(5, 2)[4], [0, 0, 0, 1, 1])
    np.testing.assert_array_equal(ref.window_mask(3, 1), np.eye(3))
    np.testing.assert_array_equal(ref.chunk_mask(7, 3)[[2, 3, 5, 6]], [[1, 1, 1, 0, 0, 0, 0], [0, 0, 0, 1, 0, 0, 0], [0, 0, 0, 1, 1, 1, 0], [0, 0, 0, 0, 0, 0, 1]])


def test_attention_terms():
    z, v, all_ = np.zeros((3, 4, 2)), np.arange(6.0).reshape(3, 2, 1), np.tril(np.ones((3, 3), bool))
    out = ref.attend(z, np.zeros((3, 2, 2)), v, all_, 1.0, sink=np.log(np.array([1.0, 3.0, 1.0, 1e-30])))
    np.testing.assert_allclose(out[2, :, 0], [(0 + 2 + 4) / 4, (0 + 2 + 4) / 6, (1 + 3 + 5) / 4, (1 + 3 + 5) / 3])
    np.testing.assert_allclose(ref.slopes(4), [0.25, 0.0625, 1 / 64, 1 / 256])
    # a cost of ln 2 a token halves the weight of every token further away
    out = ref.attend(z, np.zeros((3, 2, 2)), v, all_, 1.0, slope=np.full(4, math.log(2.0)))
    np.testing.assert_allclose(out[2, 0, 0], (0 * 0.25 + 2 * 0.5 + 4) / 1.75)
    # a cap bounds what one key can weigh
    q, k = np.full((2, 1, 1), 1e3), np.array([[[1.0]], [[0.0]]])
    out = ref.attend(q, k, np.array([[[1.0]], [[0.0]]]), np.ones((2, 2), bool), 1.0, softcap=math.log(3.0))
    np.testing.assert_allclose(out[1, 0, 0], 0.75)


def test_delta_rule():
    one, zero = np.ones((3, 1)), np.zeros((3, 1))
    k = np.tile(np.eye(2)[0], (3, 1, 1))
    v = np.arange(1.0, 4.0).reshape(3, 1, 1)
    np.testing.assert_allclose(ref.delta_rule(k, k, v, one, one)[:, 0, 0], [1, 2, 3])  # a full step replaces what the key reads
    np.testing.assert_allclose(ref.delta_rule(k, k, v, 0.5 * one, np.array([[1.0], [0], [0]]))[:, 0, 0], [1, 0.5, 0.25])
    np.testing.assert_allclose(ref.delta_rule(k, k, v, one, zero), 0.0 * v)


def test_linear_recurrence_and_filters():
    a, b = np.full((4, 1), 0.5), np.array([[8.0], [0], [0], [1]])
    np.testing.assert_allclose(ref.linear_recurrence(a, b)[:, 0], [8, 4, 2, 2])
    np.testing.assert_allclose(ref.short_conv(np.array([[1.0], [10], [100]]), np.array([[2.0, 3.0, 5.0]]))[:, 0], [5, 53, 532])
    g = ref.block_gate(np.array([[1.0, 2.0, 3.0, 4.0]]), np.array([[[0, 1.0], [0, 0]], [[0, 0], [1.0, 0]]]), np.array([[0, 1.0], [2.0, 0]]))
    np.testing.assert_allclose(g[0], ref.sigmoid(np.array([2.0, 1.0, 2.0, 3.0])))


def test_routing_within_groups():
    logit = lambda s: np.log(s / (1 - s))
    s = np.array([[0.9, 0.1, 0.1, 0.6, 0.55, 0.2, 0.3, 0.35]])  # groups of two: 1.0, 0.7, 0.75, 0.65
    w = {"router": np.eye(8)}
    r = dict(experts=8, top=2, scale=2.0, groups=dict(count=4, keep=2))
    np.testing.assert_allclose(ref.route(logit(s), w, "", r)[0], np.array([0.9, 0, 0, 0, 0.55, 0, 0, 0]) * 2.0 / 1.45)
    r["groups"]["keep"] = 4
    np.testing.assert_allclose(ref.route(logit(s), w, "", r)[0], np.array([0.9, 0, 0, 0.6, 0, 0, 0, 0]) * 2.0 / 1.5)


def test_steady_routing_is_what_it_says():
    cfg = u.config([(u.windowed_delta(), u.moe()), (u.chunked(), u.moe(experts=8, top=2, groups=4, keep=3))])
    w = u.oracle_weights(u.steady_weights(cfg, 3))
    t = np.random.default_rng(1).integers(0, cfg["vocab"], 60)
    chosen = []
    full, route = ref.forward(cfg, w, t), ref.route
    try:
        ref.route = lambda h, w_, p, r: chosen.append(route(h, w_, p, r) > 0) or route(h + np.random.default_rng(0).standard_normal(h.shape) * 0.01, w_, p, r)
        shaken = ref.forward(cfg, w, t)
    finally:
        ref.route = route
    assert all(len({tuple(r) for r in c}) > 3 for c in chosen), "the choices do not depend on the token"
    assert u.rel_rms(shaken, full).max() < BF16_LIMIT


# ---- mistakes planted in the restatement show in the outputs the GPU tests look at ----------------------------------------
def planted():
    names = ("bigram_rows", "embed", "rotate", "window_mask", "chunk_mask", "slopes", "attend", "windowed_attention", "keyed_attention", "chunked_attention",
             "short_conv", "unit", "delta_rule", "gated_delta", "block_gate", "linear_recurrence", "gated_unit", "gelu_tanh", "clamped_glu", "route", "silu", "softplus",
             "rms", "sigmoid")
    g = {n: getattr(ref, n) for n in names}

    def other_pairs(x, rot):
        n = rot["dims"]
        order = np.r_[np.arange(0, n, 2), np.arange(1, n, 2), np.arange(n, x.shape[-1])]
        return g["rotate"](x[..., np.argsort(order)], rot)[..., order]

    def rotated_all(x, rot):
        return g["rotate"](x, dict(rot, dims=x.shape[-1]))

    def read_before_write(q, k, v, decay, beta):
        S, out = np.zeros((q.shape[1], q.shape[2], v.shape[-1])), np.zeros_like(v)
        for t in range(len(q)):
            S = S * decay[t][:, None, None]
            out[t] = np.einsum("hde,hd->he", S, q[t])
            S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t])))[:, None, :]
        return out

    def fade_behind(q, k, v, decay, beta):
        return g["delta_rule"](q, k, v, np.vstack([decay[1:], decay[-1:]]), beta)

    def ungated(name):  # gates read as one half everywhere: doubled logits of zero
        return lambda h, w, p, m, *a: g[name](h, dict(w, **{p + "g": 0 * w[p + "g"]}), p, m, *a)

    def normed_values(h, w, p, m, eps):
        T, H, G = h.shape[0], m["heads"], m["kv_heads"]
        q, k = ((g["rms"](h @ w[p + n].T, eps) * w[p + n + ".norm"]).reshape(T, c, -1) for n, c in (("q", H), ("k", G)))
        o = ref.attend(ref.rotate(q, m["rot"]), ref.rotate(k, m["rot"]), k, ref.window_mask(T, m["mask"]["size"]), m["scale"])
        return (o.reshape(T, -1) * ref.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def head_norms(h, w, p, m, eps):
        T, H, G = h.shape[0], m["heads"], m["kv_heads"]
        k0 = (h @ w[p + "k"].T).reshape(T, G, -1)
        q, k = (g["rms"]((h @ w[p + n].T).reshape(T, c, -1), eps) * w[p + n + ".norm"].reshape(c, -1) for n, c in (("q", H), ("k", G)))
        o = ref.attend(ref.rotate(q, m["rot"]), ref.rotate(k, m["rot"]), k0, ref.window_mask(T, m["mask"]["size"]), m["scale"])
        return (o.reshape(T, -1) * ref.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def unnormed_input(h, w, p):
        s = ref.linear_recurrence
        try:
            ref.linear_recurrence = lambda a, b: s(a, b / np.sqrt(1 - a * a))
            return g["gated_unit"](h, w, p)
        finally:
            ref.linear_recurrence = s

    return {
        "pair row of the first token": dict(bigram_rows=lambda t, b: np.r_[int(t[0]) * b["mul_cur"] % b["buckets"], g["bigram_rows"](t, b)[1:]]),
        "pairs the other way round": dict(bigram_rows=lambda t, b: g["bigram_rows"](t, dict(b, mul_prev=b["mul_cur"], mul_cur=b["mul_prev"]))),
        "pair embedding scaled": dict(embed=lambda t, w, e: g["embed"](t, dict(w, bigram=w["bigram"] * e["scale"]), e)),
        "embedding not scaled": dict(embed=lambda t, w, e: g["embed"](t, w, dict(e, scale=1.0))),
        "rotation pairs halves": dict(rotate=other_pairs),
        "whole heads rotated": dict(rotate=rotated_all),
        "no rotation": dict(rotate=lambda x, rot: x),
        "window too wide": dict(window_mask=lambda T, n: g["window_mask"](T, n + 1)),
        "window too narrow": dict(window_mask=lambda T, n: g["window_mask"](T, n - 1)),
        "chunk too long": dict(chunk_mask=lambda T, n: g["chunk_mask"](T, n + 1)),
        "window in place of a chunk": dict(chunk_mask=lambda T, n: g["window_mask"](T, n)),
        "no cost of distance": dict(slopes=lambda H: 0 * g["slopes"](H)),
        "slopes of heads from zero": dict(slopes=lambda H: g["slopes"](H) * 2.0 ** (8.0 / H)),
        "no sink": dict(attend=lambda *a, **k: g["attend"](*a, **dict(k, sink=None))),
        "scaled sink": dict(attend=lambda q, k, v, m, s, **o: g["attend"](q, k, v, m, s, **dict(o, sink=o["sink"] * s if o.get("sink") is not None else None))),
        "no cap": dict(attend=lambda *a, **k: g["attend"](*a, **dict(k, softcap=None))),
        "no output gate (windowed)": dict(windowed_attention=ungated("windowed_attention")),
        "no output gate (keys as values)": dict(keyed_attention=ungated("keyed_attention")),
        "no output gate (chunked)": dict(chunked_attention=ungated("chunked_attention")),
        "values behind the norm": dict(keyed_attention=normed_values),
        "norms by head": dict(keyed_attention=head_norms),
        "no biases": dict(windowed_attention=lambda h, w, p, m: g["windowed_attention"](h, dict(w, **{p + n + ".b": 0 * w[p + n + ".b"] for n in "qkv"}), p, m)),
        "filter turned round": dict(short_conv=lambda x, f: g["short_conv"](x, f[:, ::-1])),
        "no unit norms": dict(unit=lambda x: x),
        "read before the write": dict(delta_rule=read_before_write),
        "decay of the next token": dict(delta_rule=fade_behind),
        "sigmoid on the delta rule's output": dict(silu=lambda x: g["sigmoid"](x)),
        "no factor 8 in the decay": dict(gated_unit=lambda h, w, p: g["gated_unit"](h, dict(w, **{p + "lam": np.log(np.expm1(g["softplus"](w[p + "lam"]) / 8))}), p)),
        "no growth of the input": dict(gated_unit=unnormed_input),
        "no input gate": dict(gated_unit=lambda h, w, p: g["gated_unit"](h, dict(w, **{p + "ri.b": w[p + "ri.b"] + 50}), p)),
        "no bias behind the filter": dict(gated_unit=lambda h, w, p: g["gated_unit"](h, dict(w, **{p + "conv.b": 0 * w[p + "conv.b"]}), p)),
        "gates turned round": dict(block_gate=lambda x, w, b: g["block_gate"](x, w.transpose(0, 2, 1), b)),
        "second branch without its gelu": dict(gelu_tanh=lambda z: z),
        "no limit": dict(clamped_glu=lambda h, w, p, limit: g["clamped_glu"](h, w, p, 1e9)),
        "no groups": dict(route=lambda h, w, p, r: g["route"](h, w, p, dict(r, groups=dict(count=1, keep=1)))),
        "weights not divided": dict(route=lambda h, w, p, r: np.where(g["route"](h, w, p, r) > 0, g["sigmoid"](h @ w[p + "router"].T) * r["scale"], 0.0)),
        "weights not scaled": dict(route=lambda h, w, p, r: g["route"](h, w, p, dict(r, scale=1.0))),
    }


@pytest.mark.parametrize("name", sorted(planted()))
def test_planted_mistakes_would_show(name):
    cfg = u.config([(u.windowed_delta(), u.dense()), (u.keyed_unit(), u.moe()), (u.chunked(), u.moe()), (u.chunked(kv_from=2), None)])
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
        assert err > BF16_LIMIT, (name, make.__name__, err)


def test_constants_of_the_stack_show():
    cfg = u.config([(u.windowed_delta(), u.dense()), (u.keyed_unit(), None), (u.chunked(), None), (u.chunked(kv_from=2, chunk=20, scale=0.3), None)])
    w = u.oracle_weights(u.weights(cfg, 8))
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 75)
    want = ref.forward(cfg, w, t)
    for change in (dict(residual_mult=1.0), dict(logit_softcap=1e9)):
        assert u.rel_rms(ref.forward(dict(cfg, **change), w, t), want).max() > 1.2 * BF16_LIMIT, change
    for i in (0, 1):
        for side in ("left_scale", "right_scale"):
            layers = [dict(L) for L in cfg["layers"]]
            layers[i]["mixer"] = dict(layers[i]["mixer"], **{side: 1.0})
            assert u.rel_rms(ref.forward(dict(cfg, layers=layers), w, t), want).max() > 0.5 * BF16_LIMIT, (i, side)


NEEDLES = {"windowed": lambda: u.windowed_delta(window=50, right=0.0), "keyed": lambda: u.keyed_unit(window=50, rot=24, base=5e5, right=0.0),
           "chunked": lambda: u.chunked(chunk=100, softcap=30.0)}


@pytest.mark.parametrize("name", sorted(NEEDLES))
def test_needle_decides(name):
    cfg = u.config([(NEEDLES[name](), None)], width=96)
    w = u.oracle_weights(u.needle_weights(cfg, 3, key_token=7))
    t = np.random.default_rng(0).integers(8, cfg["vocab"], 200)
    t[64] = 7
    blind = t.copy()
    blind[64] = 9
    err = u.rel_rms(ref.forward(cfg, w, t), ref.forward(cfg, w, blind))
    last = 99 if name == "chunked" else 64 + 49
    assert err[65:last + 1].min() > 3 * BF16_LIMIT and err[last + 1:].max() < 1e-9, (err[65:last + 1].min(), err[last + 1:].max())


def test_directory_is_recognised_by_its_config(tmp_path):
    from xfastertransformer_amd import automodel
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Duvadra"}))
    assert automodel._lib.xft_automodel_is_plan(os.fsencode(str(tmp_path)))
