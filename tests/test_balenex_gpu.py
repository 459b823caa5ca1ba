"""Balenex (attention whose window leaves block means or first tokens in sight, filters and turned values, gated linear attention beside
attention, norms in groups, biases) on the GPU against the plain restatement in oracle/balenex_ref.py: every mechanism alone, whole
models, portions, batches, page and slot reuse, borders of pages, windows and blocks, long decoding, and generation through AutoModel.
Parity unpinned: the design has no implementation elsewhere."""
import json
import os
import subprocess

import numpy as np
import pytest

import balenex_util as u
from oracle import balenex_ref as ref

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

LIMIT = {"f32": 3e-5, "bf16": 0.06}


@pytest.fixture(scope="module")
def xh():
    from xfastertransformer_amd import capi
    capi.init(0)
    return capi


def Case(xh, cfg, seed, act, slots=4, max_seq=512, max_tokens=None, pool=0, bits=None):
    bits = bits or u.weights(cfg, seed)
    return u.Case(xh, u.build_plan(xh, cfg, bits), u.oracle_weights(bits), lambda w, t: ref.forward(cfg, w, t), act, LIMIT[act], slots, max_seq, max_tokens, pool)


def tokens_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(int)


ALONE = {  # name: (layers, changes of the configuration)
    "pooled": ([(u.pooled(), None)], {}),
    "pooled_one_head": ([(u.pooled(heads=1, kv_heads=1, dim=34, vdim=6, window=20), None)], {}),
    "pooled_equal_heads": ([(u.pooled(heads=3, kv_heads=3, dim=32, vdim=32, window=64, pool=32), None)], {}),
    "blocks_of_one": ([(u.pooled(pool=1), None)], {}),
    "blocks_of_two": ([(u.pooled(pool=2, window=33), None)], {}),
    "blocks_of_sixty_four": ([(u.pooled(pool=64, window=3), None)], {}),
    "blocks_longer_than_pages": ([(u.pooled(pool=70, window=1), None)], {}),
    "windows_of_one": ([(u.pooled(window=1, pool=7), None)], {}),
    "window_beyond_the_sequence": ([(u.pooled(window=4000, pool=3), None)], {}),
    "different_blocks": ([(u.pooled(pool=3), None), (u.pooled(pool=11, window=20), None), (u.pooled(pool=3, window=5, heads=4, kv_heads=4), None)], {}),
    "pooled_wide": ([(u.pooled(heads=4, kv_heads=2, dim=200, vdim=136, scale=0.03), None)], {}),
    "pooled_very_wide": ([(u.pooled(heads=2, kv_heads=1, dim=300, vdim=264, scale=0.02), None)], {}),
    "many_heads": ([(u.pooled(heads=40, kv_heads=2, dim=64, vdim=64, scale=0.1), None)], {}),
    "odd_values": ([(u.pooled(vdim=13), None)], {}),
    "pair": ([(u.pair(), None)], {}),
    "nothing_kept": ([(u.pair(keep=0), None)], {}),
    "one_token_kept": ([(u.pair(keep=1, window=1), None)], {}),
    "more_kept_than_windows": ([(u.pair(keep=100, window=10), None)], {}),
    "everything_kept": ([(u.pair(keep=1000, window=3), None)], {}),
    "no_rotation": ([(u.pair(rot=0), None)], {}),
    "two_rotated": ([(u.pair(rot=2, dim=40, heads=6, kv_heads=1), None)], {}),
    "all_rotated": ([(u.pair(rot=20), None)], {}),
    "values_of_two": ([(u.pair(vdim=2), None)], {}),
    "wide_values": ([(u.pair(heads=4, kv_heads=2, dim=40, vdim=140), None)], {}),
    "filter_of_one": ([(u.pair(conv=1), None)], {}),
    "filter_of_two": ([(u.pair(conv=2), None)], {}),
    "long_filter": ([(u.pair(conv=7), None)], {}),
    "pair_wide": ([(u.pair(heads=4, kv_heads=2, dim=200, vdim=136, scale=0.1, rot=60), None)], {}),
    "pair_very_wide": ([(u.pair(heads=2, kv_heads=1, dim=300, vdim=270, scale=0.05, rot=200), None)], {}),
    "linear_narrow": ([(u.pair(r_heads=1, r_dim=5, r_vdim=3, rank=1), None)], {}),
    "linear_64": ([(u.pair(r_heads=2, r_dim=64, r_vdim=40, tau=1.0), None)], {}),
    "linear_100": ([(u.pair(r_heads=2, r_dim=100, r_vdim=70, tau=16.0, rank=40), None)], {}),
    "linear_128": ([(u.pair(r_heads=5, r_dim=128, r_vdim=128, tau=0.5), None)], {}),
    "linear_200": ([(u.pair(r_heads=2, r_dim=200, r_vdim=20, tau=30.0), None)], {}),
    "feed_forward": ([(u.pooled(), u.dense())], {}),
    "one_group": ([(u.pooled(), u.dense(ff=33)), (u.pair(), u.dense(ff=64))], dict(groups=1)),
    "groups_of_one": ([(u.pooled(), u.dense())], dict(width=40, groups=40, eps=0.1)),
    "groups_of_25": ([(u.pooled(), u.dense()), (u.pair(), None)], dict(width=100, groups=4)),
    "groups_of_64": ([(u.pair(), u.dense())], dict(width=320, groups=5)),
    "large_eps": ([(u.pair(), u.dense()), (u.pooled(), None)], dict(eps=0.3)),
}


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(ALONE))
def test_mechanism_alone(xh, name, act):
    """the residual behind every layer and the logits of a prompt, then token by token"""
    layers, change = ALONE[name]
    cfg = u.config(layers, **change)
    c = Case(xh, cfg, 11, act)
    t = tokens_of(cfg, 150, 1)
    streams = []
    want = ref.forward(cfg, c.w, t, streams)
    c.model.trace_residual(True)
    got = c.model.step([(0, t, list(range(len(t))))])
    tr = c.model.read_residual()
    assert tr.shape == (len(layers), len(t), cfg["width"])
    for i, s in enumerate(streams):
        c.check(tr[i], s, f"{name}: residual behind layer {i}")
    c.check(got, want, name)
    c.model.trace_residual(False)
    c.run(1, t[:40], [1], name + " token by token", want[:40])
    c.run(2, t, [70, 2, 1, 40], name + " in portions", want)
    c.run(3, t, [137, 1], name + " decoded", want)
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("shape", [(1100, 4), (1280, 5), (3000, 3), (5120, 8), (4100, 41), (9216, 9)], ids=str)
def test_norms_of_wide_rows(xh, act, shape):
    """few rows and many, groups of all kinds of sizes"""
    width, groups = shape
    cfg = u.config([(u.pooled(heads=2, kv_heads=1), None), (u.pair(heads=2, kv_heads=1, r_heads=1, r_vdim=8), None)], width=width, groups=groups, vocab=40)
    w = u.oracle_weights(u.weights(cfg, 4))
    w["embed"] *= np.exp(np.random.default_rng(1).standard_normal(groups)).repeat(width // groups)  # (groups of different lengths)
    c = Case(xh, cfg, 0, act, bits={k: u.bf16_bits(v) for k, v in w.items()})
    c.run(0, tokens_of(cfg, 110, 3), [80, 30], "wide rows")
    c.free()


@pytest.mark.parametrize("rows", [1, 5, 33, 130])
@pytest.mark.parametrize("shape", [(64, 48), (512, 320)], ids=str)
def test_gate_and_up_product_with_biases(xh, shape, rows):
    K, inter = shape
    rng = np.random.default_rng(rows)
    w = xh.f32_to_bf16_bits(rng.standard_normal((K, 2 * inter)).astype(np.float32) / K ** 0.5)
    a = xh.f32_to_bf16_bits(rng.standard_normal((rows, K)).astype(np.float32))
    b = rng.standard_normal(2 * inter).astype(np.float32)
    weight = xh.Weight(xh.W_BF16, K, 2 * inter, w, flags=xh.WF_GATEUP)
    ad, bd, out = xh.DeviceBuffer(a.nbytes), xh.DeviceBuffer(b.nbytes), xh.DeviceBuffer(rows * inter * 4)
    ad.upload(a), bd.upload(b)
    xh.gemm_gateup_silu_bias(weight, ad.ptr, rows, K, out.ptr, inter, bd.ptr, out_dtype=xh.F32)
    xh.synchronize()
    z = u.bf16_values(a) @ u.bf16_values(w) + b
    want = ref.silu(z[:, :inter]) * z[:, inter:]
    np.testing.assert_allclose(out.to_numpy(np.float32, (rows, inter)), want, rtol=2e-3, atol=2e-3)


def whole_config(**kw):
    return u.config([(u.pair(), u.dense()), (u.pooled(heads=4, kv_heads=4, dim=16, vdim=16, window=40, pool=10), u.dense(ff=72)), (u.pooled(window=21, pool=7), None),
                     (u.pair(heads=4, kv_heads=2, dim=24, vdim=16, window=65, keep=33, rot=24, conv=2, r_heads=2, r_dim=40, r_vdim=32, tau=12.0), u.dense()),
                     (u.pooled(window=64, pool=32), u.dense(ff=24)), (u.pair(window=32, keep=2, conv=3, rank=33), None)], **kw)


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("portions", [[300], [1], [2], [3, 2], [64], [63, 1, 65], [31, 33, 2, 1, 120], [17, 16, 15]], ids=str)
def test_portions(xh, act, portions):
    cfg = whole_config()
    c = Case(xh, cfg, 6, act)
    n = 300 if portions != [1] else 150
    c.run(0, tokens_of(cfg, n, 3), portions, "portions")
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_first_tokens(xh, act):
    """sequences of 1 .. 6 tokens, in a slot another sequence has used before"""
    cfg = whole_config()
    c = Case(xh, cfg, 7, act, slots=1)
    for n in range(1, 7):
        c.run(0, tokens_of(cfg, n, 40 + n), [n], f"{n} tokens")
        c.model.seq_release(0)
        c.run(0, tokens_of(cfg, n, 50 + n), [1], f"{n} tokens one by one")
        c.model.seq_release(0)
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_unequal_batches_and_reuse(xh, act):
    """Sequences come, rest, go on and end; portions of some beside single tokens of others; the pool is as small as the
    live sequences allow, so that pages and slots change hands all the time."""
    cfg = whole_config()
    slots, pool = 4, 9 * 64
    c = Case(xh, cfg, 8, act, slots=slots, max_seq=512, max_tokens=512, pool=pool)
    rng = np.random.default_rng(9)
    live, made, steps = {}, 0, 0
    while made < 14 or live:
        for s in range(slots):
            pages = sum(-(-len(q["t"]) // 64) for q in live.values())
            if s not in live and made < 14 and rng.random() < 0.7:
                n = int(rng.choice([1, 2, 5, 63, 64, 65, 130, 200]))
                if pages + -(-n // 64) > 9:
                    continue
                t = tokens_of(cfg, n, 100 + made)
                live[s] = dict(t=t, at=0, want=c.want(t))
                made += 1
        entries, expect = [], []
        for s in rng.permutation(list(live)):
            q = live[s]
            if rng.random() < 0.25:
                continue
            n = min(int(rng.choice([1, 1, 2, 3, 17, 40, 64, 90])), len(q["t"]) - q["at"])
            places = list(range(n)) if rng.random() < 0.8 else []
            entries.append((int(s), q["t"][q["at"]:q["at"] + n], places))
            if places:
                expect.append(q["want"][q["at"]:q["at"] + n])
            q["at"] += n
        if not entries:
            continue
        got = c.model.step(entries)
        if expect:
            c.check(got, np.concatenate(expect), f"step {steps}")
        steps += 1
        for s in [s for s in live if live[s]["at"] == len(live[s]["t"])]:
            c.model.seq_release(s)
            del live[s]
    assert c.model.pool_pages() == (9, 9)
    c.free()


@pytest.mark.parametrize("pool", [1, 3, 64, 100])
def test_pages_of_block_means_suffice(xh, pool):
    """four sequences that fill the page pool to the last token, whatever their lengths"""
    cfg = u.config([(u.pooled(heads=2, kv_heads=1, window=6, pool=pool), None)])
    c = Case(xh, cfg, 3, "f32", slots=4, max_seq=640, max_tokens=640, pool=640)
    for lengths in ((448, 64, 64, 64), (640,), (192, 192, 192, 64), (128, 192, 1, 256)):
        for s, n in enumerate(lengths):
            t = tokens_of(cfg, n, 30 + s)
            c.run(s, t, [n - 1, 1] if n > 1 else [1], f"{lengths}: {n} tokens")
        for s in range(len(lengths)):
            c.model.seq_release(s)
    c.free()


def test_a_batch_gives_what_each_alone_gives(xh):
    """single tokens, short and long portions in one step, beyond the few-row products: the same logits as one by one"""
    cfg = whole_config()
    for act, limit in (("f32", 1e-5), ("bf16", 0.03)):
        c = Case(xh, cfg, 16, act, slots=4)
        seqs = [tokens_of(cfg, n, 20 + n) for n in (230, 70, 41, 9)]
        cut = [165, 69, 40, 2]
        alone = [np.concatenate([c.model.step([(s, t[:k], list(range(k)))]), c.model.step([(s, t[k:], list(range(len(t) - k)))])])
                 for s, (t, k) in enumerate(zip(seqs, cut))]
        for s in range(4):
            c.model.seq_release(s)
        order = [2, 0, 3, 1]
        got = [c.model.step([(s, seqs[s][:cut[s]], list(range(cut[s]))) for s in order]),
               c.model.step([(s, seqs[s][cut[s]:], list(range(len(seqs[s]) - cut[s]))) for s in order])]
        want = [np.concatenate([alone[s][:cut[s]] for s in order]), np.concatenate([alone[s][cut[s]:] for s in order])]
        for g, w in zip(got, want):
            assert u.rel_rms(g, w).max() < limit
        c.free()


SHAPES = {  # the attention kernels' forms: query / key size of a head (values alike)
    "128": dict(heads=4, kv_heads=2, dim=128),
    "64": dict(heads=16, kv_heads=2, dim=64),
    "odd": dict(heads=6, kv_heads=3, dim=90),
    "small": dict(heads=5, kv_heads=5, dim=20),
    "large": dict(heads=2, kv_heads=1, dim=250),
    "larger": dict(heads=1, kv_heads=1, dim=290),
}
SPAN, KEEP, POOL = 75, 40, 4


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("shape", sorted(SHAPES))
@pytest.mark.parametrize("kind", ["first", "pooled"])
def test_needle(xh, kind, shape, act):
    """One key decides every later answer that sees it.  It is planted at borders of pages, blocks and the kept tokens and elsewhere, and read
    far away, just inside and just outside the window, when its block is about to be seen, in prompts, in portions and by decoded tokens."""
    s = SHAPES[shape]
    d = s["dim"]
    if kind == "first":
        m = u.pair(vdim=d, rot=d // 4 * 2, base=5e5, window=SPAN, keep=KEEP, scale=8.0 / d, **s)
    else:
        m = u.pooled(vdim=d, window=SPAN, pool=POOL, scale=40.0 / d, **s)
    cfg = u.config([(m, None)], width=96)
    bits = u.needle_weights(cfg, 3, key_token=7)
    c = Case(xh, cfg, 0, act, slots=3, max_seq=448, bits=bits)
    for place in (0, 31, 39, 40, 63, 64, 75, 102):
        t = np.random.default_rng(place).integers(8, cfg["vocab"], 260)
        t[place] = 7
        want = c.want(t)
        t2 = t.copy()
        t2[place] = 9
        shows = u.rel_rms(want, c.want(t2))
        last = place + SPAN - 1  # the last position whose window has the needle
        back = place // POOL * POOL + POOL - 1 + SPAN if kind == "pooled" else last + 1 if place < KEEP else 260  # the first that sees it again
        inside = [i for i in range(place + 1, 260) if i <= last or i >= back]
        outside = [i for i in range(last + 1, min(back, 260))]
        assert shows[inside].min() > 1.5 * LIMIT["bf16"] and (not outside or shows[outside].max() < 1e-9), "the needle does not show"
        c.run(0, t, [260], f"{kind} needle at {place}, prompt", want)
        c.run(1, t, [place + 20, 2, 1, 1, 1, 7], f"{kind} needle at {place}, portions", want)
        c.run(2, t[:last + 8], [max(last - 2, 1), 1], f"{kind} needle at {place}, decoded over the edge", want)
        for i in range(3):
            c.model.seq_release(i)
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_states_remember(xh, act):
    """Linear attention that hardly fades carries the first tokens through hundreds of others, prompt, portions and decoding; what the
    sequence began with shows at its end."""
    cfg = u.config([(u.pair(tau=200.0, keep=0, window=5, r_vdim=12), None)])
    w = u.oracle_weights(u.weights(cfg, 5))
    w["l0.mix.right.a2.b"][:] = 6.0
    w["l0.mix.left.out"][:] = 0.0
    c = Case(xh, cfg, 0, act, bits={k: u.bf16_bits(v) for k, v in w.items()})
    t = tokens_of(cfg, 400, 6)
    want = c.want(t)
    t2 = t.copy()
    t2[:50] = tokens_of(cfg, 50, 7)
    assert u.rel_rms(want, c.want(t2))[-1] > LIMIT["bf16"]
    c.run(0, t, [400], "prompt", want)
    c.run(1, t, [130, 2, 65, 1, 1, 100, 64], "portions", want)
    c.run(2, t, [370, 1], "decoded", want)
    c.free()


def test_split_contexts_and_long_portions(xh):
    """long contexts over many parts of the chip, decoded, in short and in long portions"""
    cfg = u.config([(u.pooled(heads=8, kv_heads=2, dim=128, vdim=128, scale=0.05, window=300, pool=2), None),
                    (u.pair(heads=20, kv_heads=2, dim=64, vdim=128, scale=0.3, window=500, keep=400, r_heads=2, r_dim=128, r_vdim=64), None),
                    (u.pooled(heads=8, kv_heads=1, dim=64, vdim=64, window=700, pool=16, scale=0.1), None)], width=128, groups=4)
    c = Case(xh, cfg, 12, "bf16", slots=3, max_seq=1600, max_tokens=1600)
    t = tokens_of(cfg, 1500, 6)
    want = c.want(t)
    c.run(0, t, [1100, 1, 1, 2, 5, 16, 1, 17, 56, 99, 1, 1, 1, 200], "long", want)
    for s in (1, 2):
        c.model.step([(s, t[:1200 + s], [])])
    got = c.model.step([(1, t[1201:1202], [0]), (2, t[1202:1205], [0, 1, 2])])
    c.check(got, want[[1201, 1202, 1203, 1204]], "side by side")
    got = c.model.step([(1, t[1202:1302], [0, 99]), (2, t[1205:1206], [0])])
    c.check(got, want[[1202, 1301, 1205]], "a long portion beside a token")
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_long_decoding(xh, act):
    """greedy decoding by graph replay: every step's chosen ids and the last logits, then the same steps launched one by one"""
    cfg = whole_config()
    c = Case(xh, cfg, 13, act, slots=2, max_seq=400, max_tokens=256)
    prompts = np.stack([tokens_of(cfg, 30, 60), tokens_of(cfg, 30, 61)]).astype(np.int32)
    runs = []
    for graph in (True, False):
        c.model.use_graph(graph)
        first, logits = c.model.prefill(prompts, want_logits=True)
        for b in range(2):
            c.check(logits[b:b + 1], c.want(prompts[b])[-1:], "prompt")
        ids = [first] + list(c.model.decode(170, 2)) + list(c.model.decode(70, 2))
        runs.append((np.stack(ids), c.model.logits(2)))
    np.testing.assert_array_equal(runs[0][0], runs[1][0])
    np.testing.assert_array_equal(runs[0][1], runs[1][1])
    ids = runs[0][0]
    for b in range(2):
        full = np.concatenate([prompts[b], ids[:-1, b]])
        want = c.want(full)
        for i, row in enumerate(want[29:]):
            assert row.max() - row[ids[i, b]] <= 3 * c.limit * want.std(), f"sequence {b}, step {i}"
        c.check(runs[0][1][b:b + 1], want[-1:], f"sequence {b}: logits behind 240 decoded tokens")
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_many_sequences_decode_together(xh, act):
    """more sequences than the few-row products take, by graph replay"""
    cfg = whole_config()
    n = 45
    c = Case(xh, cfg, 18, act, slots=n, max_seq=64, max_tokens=n * 17)
    prompts = np.stack([tokens_of(cfg, 17, 200 + i) for i in range(n)]).astype(np.int32)
    first, _ = c.model.prefill(prompts, want_logits=True)
    ids = [first] + list(c.model.decode(30, n))
    logits = c.model.logits(n)
    for b in range(n):
        full = np.concatenate([prompts[b], np.stack(ids)[:-1, b]])
        c.check(logits[b:b + 1], c.want(full)[-1:], f"sequence {b}")
    c.free()


def test_slots_that_sit_out(xh):
    cfg = whole_config()
    c = Case(xh, cfg, 14, "f32", slots=3, max_seq=256)
    seqs = [list(tokens_of(cfg, n, 70 + n)) for n in (20, 133, 5)]
    for s, t in enumerate(seqs):
        c.model.seq_prefill(s, t)
    for rows in ([2], [0, 2], [1], [2, 1], [0], [0, 1, 2]):
        for r in rows:
            i = int(c.want(seqs[r])[-1].argmax())
            c.model.seq_set_next_id(r, i)
            seqs[r].append(i)
        c.model.seq_decode(rows)
        for r in rows:
            c.check(c.model.seq_logits(r)[None], c.want(seqs[r])[-1:], f"slot {r} of {rows}")
    # a copy of a slot goes on by itself: pages, block means, filters' inputs, states
    c.model.seq_reorder([2, 0], [1, 1], 0, 0)
    for r in (0, 2):
        seqs[r] = list(seqs[1])
    for step in range(14):
        for r in range(3):
            c.model.seq_set_next_id(r, 3 + r + step)
            seqs[r].append(3 + r + step)
        c.model.seq_decode([0, 1, 2])
        for r in range(3):
            c.check(c.model.seq_logits(r)[None], c.want(seqs[r])[-1:], f"copied slot {r}, step {step}")
    c.model.seq_reorder([0, 1], [1, 0], 0, 0)
    seqs[0], seqs[1] = seqs[1], seqs[0]
    for r in range(3):
        c.model.seq_set_next_id(r, 9)
        seqs[r].append(9)
    c.model.seq_decode([0, 1, 2])
    for r in range(3):
        c.check(c.model.seq_logits(r)[None], c.want(seqs[r])[-1:], f"swapped slot {r}")
    c.free()


def test_broken_plans_are_refused(xh):
    layers, _ = u.plan_layers(u.config([(u.pooled(), u.dense()), (u.pair(), None)]))
    attention, left, right = layers
    for change in (dict(heads=5), dict(window=0), dict(pool=-1), dict(keep_first=3), dict(chunk=4), dict(distance_bias=1), dict(qk_norm=4), dict(kv_from=1), dict(dim=600),
                   dict(experts=2, top=1, expert_inter=8), dict(result_norm=1), dict(glu_alpha=1.7)):
        with pytest.raises(xh.XftHipError):
            xh.Plan(72, 90, [dict(attention, **change)], norm_groups=3, **u.STACK)
    for bad in ([left], [right], [left, dict(right, result_norm=0)], [left, dict(right, tau=0.0)], [left, dict(right, decay_rank=0)], [left, dict(right, dim=300)],
                [dict(left, vdim=13), right], [dict(left, qk_norm=2), right], [dict(left, key_values=1), right], [left, right, dict(attention, pool=0, kv_from=1)],
                [left, dict(right, inter=8)]):
        with pytest.raises(xh.XftHipError):
            xh.Plan(72, 90, bad, norm_groups=3, **u.STACK)
    for stack in (dict(u.STACK, norm_groups=5), dict(u.STACK, norm_groups=-1), dict(block=0, norm=0, norm_groups=3), dict(block=1, norm=2, norm_groups=3)):
        with pytest.raises(xh.XftHipError):
            xh.Plan(72, 90, [attention], **stack)
    cfg = u.config([(u.pair(), u.dense()), (u.pooled(), None)])
    bits = u.weights(cfg, 1)
    for name in ("l0.norm2b", "l0.mlp.up.b", "l0.mlp.down.b", "l0.mix.left.k.conv", "l0.mix.left.q.norm", "l0.mix.right.out", "l0.mix.right.a2.b", "l1.mix.o.b"):
        with pytest.raises(xh.XftHipError, match=name.split(".")[-1]):
            u.build_plan(xh, cfg, {k: v for k, v in bits.items() if k != name})


# ---- through the framework's own entry points -----------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dir(tmp_path_factory):
    cfg = whole_config()
    bits = u.weights(cfg, 21)
    path = str(tmp_path_factory.mktemp("plan") / "model")
    u.write_model(path, cfg, bits)
    return path, cfg, u.oracle_weights(bits)


def greedy(cfg, w, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(ref.forward(cfg, w, t)[-1].argmax()))
    return t


def test_generate(xh, model_dir):
    from xfastertransformer_amd.automodel import AutoModel
    path, cfg, w = model_dir
    m = AutoModel.from_pretrained(path, "fp32")
    assert m.vocab_size == cfg["vocab"]
    prompts = [list(tokens_of(cfg, 17, 80)), list(tokens_of(cfg, 17, 81))]
    expect = [greedy(cfg, w, p, 53) for p in prompts]
    out = m.generate(np.array(prompts, np.int32), max_length=70)
    np.testing.assert_array_equal(out, expect)
    out = m.generate(np.array(prompts[:1], np.int32), max_length=30, num_beams=3)
    assert out.shape[1] >= 30 and out[0, :17].tolist() == prompts[0]
    out = m.generate(np.array(prompts, np.int32), max_length=30, do_sample=True, top_k=5)
    assert out.shape == (2, 30) and out.max() < cfg["vocab"]
    # sequences by id, of different lengths, stepping and ending independently
    a, b = m.set_input_cb([prompts[0], prompts[1][:5]], max_length=40)
    got = {a: [], b: []}
    for i, x in zip((a, b), m.forward_cb()):
        got[i].append(x)
    for ids in ([a, b], [b], [a], [a, b]):
        m.set_input_cb(seq_ids=ids, max_length=40)
        for i, x in zip(ids, m.forward_cb()):
            got[i].append(x)
    assert prompts[0] + got[a] == expect[0][:17 + 4]
    assert prompts[1][:5] + got[b] == greedy(cfg, w, prompts[1][:5], 4)
    m.free_seqs([a, b])
    m.free()
    m = AutoModel.from_pretrained(path, "bf16")
    out = m.generate(np.array(prompts, np.int32), max_length=40)
    for b in range(2):
        want = ref.forward(cfg, w, out[b, :-1])[16:]
        for i, row in enumerate(want):
            assert row.max() - row[out[b, 17 + i]] <= 3 * LIMIT["bf16"] * want.std()
    m.free()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(xh, model_dir, tmp_path, dtype):
    path, cfg, w = model_dir
    seqs = {"a": tokens_of(cfg, 70, 90), "b": tokens_of(cfg, 9, 91), "c": tokens_of(cfg, 66, 92), "d": tokens_of(cfg, 3, 93), "e": tokens_of(cfg, 80, 94)}
    plan = [[("a", 60), ("b", 3)], [("b", 1), ("c", 30), ("a", 1)], [("d", 3), ("b", 5), ("a", 2)], [("e", 80), ("c", 36)], [("a", 7)]]
    at, lines, expect = {k: 0 for k in seqs}, [], {}
    for n, step in enumerate(plan):
        entries, rows, end = [], [], []
        for k, c in step:
            entries.append(dict(id=k, tokens=seqs[k][at[k]:at[k] + c].tolist(), want=[0, c - 1] if n != 1 else []))
            rows += [ref.forward(cfg, w, seqs[k])[[at[k], at[k] + c - 1]]] if n != 1 else []
            at[k] += c
            if at[k] == len(seqs[k]):
                end.append(k)
        lines.append(json.dumps(dict(step=n, entries=entries, end=end)))
        if rows:
            expect[n] = np.concatenate(rows)
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "384"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done %d" % n for n in range(len(plan))]
    assert not (tmp_path / "1.f32").exists()
    for n, want in expect.items():
        got = np.fromfile(tmp_path / ("%d.f32" % n), "<f4").reshape(-1, cfg["vocab"])
        assert u.rel_rms(got, want).max() < LIMIT["f32" if dtype == "float32" else "bf16"]
