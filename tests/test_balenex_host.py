"""The plain restatement of Balenex held against closed forms; what the GPU tests' inputs would show, with mistakes planted in the
restatement; and the parts of the loader that need no device."""
import json
import math
import os

import numpy as np
import pytest

import balenex_util as u
from oracle import balenex_ref as ref

BF16_LIMIT = 0.06  # of the GPU tests


def test_norm_in_groups():
    x = np.array([[3.0, 4.0, 0.0, 2.0]])
    np.testing.assert_allclose(ref.group_rms(x, np.array([1.0, 2.0, 3.0, 4.0]), 2, 0.0)[0], [3 / math.sqrt(12.5), 8 / math.sqrt(12.5), 0, 8 / math.sqrt(2)])
    np.testing.assert_allclose(ref.group_rms(x, np.ones(4), 1, 0.5), ref.rms(x, 0.5))
    np.testing.assert_allclose(ref.rms(np.zeros((1, 3)), 1e-5), 0.0)


def test_rotation():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal(14), rng.standard_normal(14)
    at = lambda x, p, s=1.0: ref.rotate(np.tile(x, (p + 1, 1, 1)), 10, 300.0, s)[p, 0]
    np.testing.assert_allclose(at(q, 11) @ at(k, 4), at(q, 107) @ at(k, 100), rtol=1e-10)  # only the distance counts
    np.testing.assert_array_equal(at(q, 5)[10:], q[10:])
    np.testing.assert_allclose(at(q, 3)[[0, 5]], [q[0] * math.cos(3) - q[5] * math.sin(3), q[5] * math.cos(3) + q[0] * math.sin(3)])
    np.testing.assert_allclose(at(at(q, 7), 7, -1.0), q)
    # a value that only its own position sees comes back as it was
    v = rng.standard_normal((9, 1, 6))
    np.testing.assert_allclose(ref.rotate(ref.attend(v, v, ref.rotate(v, 6, 50.0), np.eye(9, dtype=bool), 1.0), 6, 50.0, -1.0), v)


def test_masks():
    np.testing.assert_array_equal(ref.window_mask(5, 2)[4], [0, 0, 0, 1, 1])
    np.testing.assert_array_equal(ref.kept_window_mask(6, 2, 2)[[0, 1, 2, 5]], [[1, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0], [1, 1, 0, 0, 1, 1]])
    m = ref.block_mask(12, 4, 3, 4)  # block b is seen from position 3 b + 6 on
    np.testing.assert_array_equal(m.argmax(0)[:2], [6, 9])
    assert m[11].tolist() == [True, True, False, False] and not m[5].any()
    np.testing.assert_allclose(ref.block_means(np.arange(8.0).reshape(8, 1, 1), 3)[:, 0, 0], [1, 4])


def test_tokens_and_blocks_share_a_softmax():
    z, v = np.zeros((7, 1, 2)), np.arange(7.0).reshape(7, 1, 1)
    keys, values = (np.concatenate([x, ref.block_means(x, 2)]) for x in (z, v))
    out = ref.attend(z, keys, values, np.concatenate([ref.window_mask(7, 3), ref.block_mask(7, 3, 2, 3)], 1), 1.0)
    # position 6 sees tokens 4, 5, 6 and the blocks (0, 1) and (2, 3); position 5 tokens 3, 4, 5 and the block (0, 1)
    np.testing.assert_allclose(out[[5, 6], 0, 0], [(3 + 4 + 5 + 0.5) / 4, (4 + 5 + 6 + 0.5 + 2.5) / 5])


def test_linear_attention_and_filters():
    one = np.ones((4, 1, 1))
    v = np.array([8.0, 0, 0, 1]).reshape(4, 1, 1)
    np.testing.assert_allclose(ref.linear_attention(one, one, v, 0.5 * one)[:, 0, 0], [8, 4, 2, 2])
    q, k = np.tile([[[0.0, 1.0]]], (2, 1, 1)), np.tile([[[3.0, 5.0]]], (2, 1, 1))
    alpha = np.tile([[[1.0, 0.25]]], (2, 1, 1))
    np.testing.assert_allclose(ref.linear_attention(q, k, np.array([4.0, 0.0]).reshape(2, 1, 1), alpha)[:, 0, 0], [20, 5])  # a decay a key channel
    w = {"a1": np.eye(1), "a2": np.zeros((1, 1)), "a2.b": np.array([math.log(3.0)])}
    np.testing.assert_allclose(ref.decays(np.ones((1, 1)), w, "", 2.0), math.sqrt(0.75))
    np.testing.assert_allclose(ref.short_conv(np.array([[1.0], [10], [100]]), np.array([[2.0, 3.0, 5.0]]))[:, 0], [5, 53, 532])


def test_results_of_a_pair():
    w = {"left.out": np.array([1.0, 2.0]), "right.out": np.array([3.0, 1.0])}
    np.testing.assert_allclose(ref.pair(np.array([[5.0, 5.0]]), np.array([[0.1, -0.1]]), w, "", 0.0), [[2.0, 0.5]])


# ---- mistakes planted in the restatement show in the outputs the GPU tests look at ----------------------------------------
def planted():
    names = ("group_rms", "rms", "project", "short_conv", "rotate", "kept_window_mask", "window_mask", "block_mask", "block_means", "attend", "filtered_attention",
             "decays", "linear_attention", "gated_linear", "pair", "pooled_attention", "feed_forward", "silu")
    g = {n: getattr(ref, n) for n in names}

    def other_pairs(x, dims, base, sign=1.0):
        order = np.r_[np.arange(0, dims, 2), np.arange(1, dims, 2), np.arange(dims, x.shape[-1])]
        return g["rotate"](x[..., order], dims, base, sign)[..., np.argsort(order)]

    def rotations(**kw):  # rotate() with the whole head turned (a value) or not
        def f(x, dims, base, sign=1.0):
            kind = "back" if sign < 0 else "value" if dims == x.shape[-1] else "key"
            return kw[kind](x, dims, base, sign) if kind in kw else g["rotate"](x, dims, base, sign)
        return f

    def without(name, *leaves):
        return lambda h, w, p, *a: g[name](h, dict(w, **{p + n: 0 * w[p + n] for n in leaves}), p, *a)

    def read_before_write(q, k, v, alpha):
        return g["linear_attention"](q, k, v, alpha) - (q * k).sum(-1, keepdims=True) * v

    def fade_behind(q, k, v, alpha):
        return g["linear_attention"](q, k, v, np.concatenate([alpha[1:], alpha[-1:]]))

    def sums_of_blocks(x, P):
        return g["block_means"](x, P) * P

    def means_first(h, w, p, m, eps):  # keys normed behind the mean
        r = ref.block_means
        try:
            ref.block_means = lambda x, P: g["rms"](r(x, P), eps) if x.shape[-1] == m["dim"] else r(x, P)
            return g["pooled_attention"](h, w, p, m, eps)
        finally:
            ref.block_means = r

    def two_softmaxes(q, k, v, mask, scale):
        T = q.shape[0]
        if k.shape[0] == T:
            return g["attend"](q, k, v, mask, scale)
        near, far = g["attend"](q, k[:T], v[:T], mask[:, :T], scale), np.zeros((T, q.shape[1], v.shape[-1]))
        some = mask[:, T:].any(1)
        if some.any():
            far[some] = g["attend"](q[some], k[T:], v[T:], mask[some, T:], scale)
        return near + far

    def plain_queries(h, w, p, m, eps):
        r, seen = ref.rms, []
        try:
            ref.rms = lambda x, e: seen.append(1) or (x if len(seen) == 1 else r(x, e))
            return g["pooled_attention"](h, w, p, m, eps)
        finally:
            ref.rms = r

    return {
        "norms over the whole row": dict(group_rms=lambda x, w, groups, eps: g["group_rms"](x, w, 1, eps)),
        "norms in more groups": dict(group_rms=lambda x, w, groups, eps: g["group_rms"](x, w, 2 * groups, eps)),
        "norms about one": dict(group_rms=lambda x, w, groups, eps: g["group_rms"](x, 1.0 + w, groups, eps)),
        "eps outside the root": dict(rms=lambda x, eps: x / (np.sqrt((x * x).mean(-1, keepdims=True)) + 30 * math.sqrt(eps))),
        "no biases": dict(project=lambda h, w, n: h @ w[n].T),
        "no bias on the output projection": dict(pooled_attention=without("pooled_attention", "o.b")),
        "no biases on keys": dict(filtered_attention=without("filtered_attention", "k.b")),
        "no bias on the feed-forward's gate": dict(feed_forward=without("feed_forward", "gate.b")),
        "no bias behind the feed-forward": dict(feed_forward=without("feed_forward", "down.b")),
        "filter turned round": dict(short_conv=lambda x, f: g["short_conv"](x, f[:, ::-1])),
        "no filter": dict(short_conv=lambda x, f: x * f[:, -1]),
        "a silu behind the filter": dict(short_conv=lambda x, f: ref.silu(g["short_conv"](x, f))),
        "bias in front of the first token": dict(short_conv=lambda x, f: g["short_conv"](np.concatenate([x[:1]] * (f.shape[1] - 1) + [x]), f)[f.shape[1] - 1:]),
        "rotation of neighbours": dict(rotate=rotations(key=other_pairs)),
        "whole heads rotated": dict(rotate=rotations(key=lambda x, dims, base, s: g["rotate"](x, x.shape[-1], base, s))),
        "no rotation": dict(rotate=rotations(key=lambda x, *a: x)),
        "values not rotated": dict(rotate=rotations(value=lambda x, *a: x)),
        "outputs not turned back": dict(rotate=rotations(back=lambda x, *a: x)),
        "neither": dict(rotate=rotations(value=lambda x, *a: x, back=lambda x, *a: x)),
        "values by neighbours": dict(rotate=rotations(value=other_pairs, back=other_pairs)),
        "values by the keys' frequencies": dict(rotate=rotations(value=lambda x, d, b, s: g["rotate"](x, d, b ** 2, s), back=lambda x, d, b, s: g["rotate"](x, d, b ** 2, s))),
        "window too wide": dict(kept_window_mask=lambda T, n, k: g["kept_window_mask"](T, n + 1, k)),
        "window too narrow": dict(kept_window_mask=lambda T, n, k: g["kept_window_mask"](T, n - 1, k)),
        "one more first token": dict(kept_window_mask=lambda T, n, k: g["kept_window_mask"](T, n, k + 1 if k else 0)),
        "one first token less": dict(kept_window_mask=lambda T, n, k: g["kept_window_mask"](T, n, max(k - 1, 0))),
        "no first tokens": dict(kept_window_mask=lambda T, n, k: g["kept_window_mask"](T, n, 0)),
        "blocks a token early": dict(block_mask=lambda T, n, P, s: g["block_mask"](T, n, P, s - 1)),
        "blocks a token late": dict(block_mask=lambda T, n, P, s: g["block_mask"](T, n, P, s + 1)),
        "no blocks": dict(block_mask=lambda T, n, P, s: np.zeros((T, n), bool)),
        "sums of blocks": dict(block_means=sums_of_blocks),
        "blocks begin a token late": dict(block_means=lambda x, P: g["block_means"](np.concatenate([x[1:], x[-1:]]), P)),
        "keys normed behind their mean": dict(pooled_attention=means_first),
        "a softmax for tokens, one for blocks": dict(attend=two_softmaxes),
        "queries not normed": dict(pooled_attention=plain_queries),
        "read before the write": dict(linear_attention=read_before_write),
        "decay of the next token": dict(linear_attention=fade_behind),
        "no root of the decays": dict(decays=lambda h, w, p, tau: g["decays"](h, w, p, 1.0)),
        "no bias in the decays": dict(decays=lambda h, w, p, tau: g["decays"](h, dict(w, **{p + "a2.b": 0 * w[p + "a2.b"]}), p, tau)),
        "one decay a head": dict(linear_attention=lambda q, k, v, a: g["linear_attention"](q, k, v, np.broadcast_to(a.mean(-1, keepdims=True), a.shape))),
        "no gate": dict(silu=lambda x: np.ones_like(x)),
        "a sigmoid for a silu": dict(silu=ref.sigmoid),
        "results not normed": dict(pair=lambda a, b, w, p, eps: 0.5 * (a * w[p + "left.out"] + b * w[p + "right.out"])),
        "results normed together": dict(pair=lambda a, b, w, p, eps: 0.5 * (a * w[p + "left.out"] + b * w[p + "right.out"]) / np.sqrt((np.r_["1", a, b] ** 2).mean(-1, keepdims=True))),
        "results in groups": dict(pair=lambda a, b, w, p, eps: 0.5 * (g["group_rms"](a, w[p + "left.out"], 3, eps) + g["group_rms"](b, w[p + "right.out"], 3, eps))),
    }


@pytest.mark.parametrize("name", sorted(planted()))
def test_planted_mistakes_would_show(name):
    second = u.pooled(window=4, pool=2, scale=0.1) if name.startswith("blocks a token") else u.pooled()
    cfg = u.config([(u.pair(), u.dense()), (second, u.dense()), (u.pair(window=12, conv=3), None)], eps=2e-3 if name.startswith("eps") else 1e-5)
    w = u.oracle_weights(u.weights(cfg, 6))
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 150)
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
    assert err > BF16_LIMIT, (name, err)


def test_half_the_sum_shows_where_nothing_norms_it():
    """(the norm behind the mixer takes a factor of the pair out again: only eps can tell)"""
    cfg = u.config([(u.pair(), None)], eps=0.5)
    w = u.oracle_weights(u.weights(cfg, 6))
    t = np.random.default_rng(2).integers(0, cfg["vocab"], 40)
    want, pair = ref.forward(cfg, w, t), ref.pair
    try:
        ref.pair = lambda *a: 2.0 * pair(*a)
        assert u.rel_rms(ref.forward(cfg, w, t), want).max() > BF16_LIMIT
    finally:
        ref.pair = pair


def needle_case(kind, **kw):
    """configuration, and the positions that see a needle at `place` (of a sequence of n tokens)"""
    if kind == "first":
        m = u.pair(window=40, keep=kw["keep"], rot=10, base=5e5)
        sees = lambda place, n: [i for i in range(place + 1, n) if i - place < 40 or place < kw["keep"]]
    else:
        m = u.pooled(window=40, pool=kw["pool"], scale=2.5)
        end = lambda place: place // kw["pool"] * kw["pool"] + kw["pool"] - 1
        sees = lambda place, n: [i for i in range(place + 1, n) if i - place < 40 or end(place) <= i - 40]
    return u.config([(m, None)], width=96), sees


@pytest.mark.parametrize("kind,kw", [("first", dict(keep=20)), ("first", dict(keep=0)), ("pooled", dict(pool=2)), ("pooled", dict(pool=4))], ids=str)
def test_needle_decides(kind, kw):
    cfg, sees = needle_case(kind, **kw)
    w = u.oracle_weights(u.needle_weights(cfg, 3, key_token=7))
    for place in (5, 19, 20, 64):
        t = np.random.default_rng(0).integers(8, cfg["vocab"], 200)
        t[place] = 7
        blind = t.copy()
        blind[place] = 9
        err = u.rel_rms(ref.forward(cfg, w, t), ref.forward(cfg, w, blind))
        seen = sees(place, 200)
        rest = [i for i in range(200) if i not in seen and i != place]
        assert err[seen].min() > 1.5 * BF16_LIMIT and err[rest].max() < 1e-9, (place, err[seen].min(), err[rest].max())


def test_directory_is_recognised_by_its_config(tmp_path):
    from xfastertransformer_amd import automodel
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Balenex"}))
    assert automodel._lib.xft_automodel_is_plan(os.fsencode(str(tmp_path)))
