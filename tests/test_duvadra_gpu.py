"""Duvadra (chunked, windowed and key-valued attention over pages, a gated delta rule and a gated linear recurrence beside attention,
experts routed within groups, token-pair embeddings) on the GPU against the plain restatement in oracle/duvadra_ref.py: every mechanism
alone, whole models, portions, batches, page and slot reuse, borders of pages, windows and chunks, long decoding, and generation through
AutoModel.  Parity unpinned: the design has no implementation elsewhere."""
import json
import os
import subprocess

import numpy as np
import pytest

import duvadra_util as u
from oracle import duvadra_ref as ref

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

LIMIT = {"f32": 3e-5, "bf16": 0.06}


@pytest.fixture(scope="module")
def xh():
    from xfastertransformer_amd import capi
    capi.init(0)
    return capi


def Case(xh, cfg, seed, act, slots=4, max_seq=512, max_tokens=None, pool=0, bits=None):
    bits = bits or (u.weights if act == "f32" else u.steady_weights)(cfg, seed)
    return u.Case(xh, u.build_plan(xh, cfg, bits), u.oracle_weights(bits), lambda w, t: ref.forward(cfg, w, t), act, LIMIT[act], slots, max_seq, max_tokens, pool)


def tokens_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(int)


ALONE = {  # name: (layers, changes of the configuration)
    "chunked": ([(u.chunked(), None)], {}),
    "chunked_one_head": ([(u.chunked(heads=1, kv_heads=1, dim=34, vdim=6, scale=1.0), None)], {}),
    "chunked_equal_heads": ([(u.chunked(heads=3, kv_heads=3, dim=32, vdim=32, chunk=64), None)], {}),
    "chunks_of_one": ([(u.chunked(chunk=1), None)], {}),
    "chunk_beyond_the_sequence": ([(u.chunked(chunk=4000, softcap=50.0), None)], {}),
    "chunked_wide": ([(u.chunked(heads=4, kv_heads=2, dim=200, vdim=136, scale=0.1), None)], {}),
    "chunked_very_wide": ([(u.chunked(heads=2, kv_heads=1, dim=300, vdim=264, scale=0.1), None)], {}),
    "many_heads": ([(u.chunked(heads=40, kv_heads=2, dim=64, vdim=64, scale=0.2), None)], {}),
    "shared_keys": ([(u.chunked(), None), (u.windowed_delta(), None), (u.chunked(kv_from=0, chunk=11, scale=0.8, softcap=3.0), u.dense()), (u.chunked(kv_from=0), None)], {}),
    "windowed_delta": ([(u.windowed_delta(), None)], {}),
    "windowed_only": ([(u.windowed_delta(right=0.0), None)], {}),
    "windows_of_one": ([(u.windowed_delta(window=1, right=0.0), None)], {}),
    "delta_only": ([(u.windowed_delta(left=0.0), None)], {}),
    "delta_equal_heads": ([(u.windowed_delta(heads=2, kv_heads=1, r_heads=3, r_kv_heads=3, r_dim=32, r_vdim=32, conv=4, left=0.0, right=-1.0), None)], {}),
    "delta_no_filter": ([(u.windowed_delta(conv=1, left=0.0), None)], {}),
    "delta_two_taps": ([(u.windowed_delta(conv=2, left=0.0), None)], {}),
    "delta_long_filter": ([(u.windowed_delta(conv=7, left=0.0), None)], {}),
    "delta_wide": ([(u.windowed_delta(r_heads=2, r_kv_heads=1, r_dim=100, r_vdim=150, left=0.0), None)], {}),
    "delta_wider": ([(u.windowed_delta(r_heads=2, r_kv_heads=2, r_dim=200, r_vdim=40, conv=4, left=0.0), None)], {}),
    "keyed_unit": ([(u.keyed_unit(), None)], {}),
    "keyed_only": ([(u.keyed_unit(right=0.0), None)], {}),
    "keyed_all_rotated": ([(u.keyed_unit(rot=24, right=0.0), None)], {}),
    "keyed_two_rotated": ([(u.keyed_unit(heads=6, kv_heads=1, dim=40, rot=2, right=0.0), None)], {}),
    "keyed_wide": ([(u.keyed_unit(heads=9, kv_heads=3, dim=272, rot=100, scale=0.05, right=0.0), None)], {}),
    "unit_only": ([(u.keyed_unit(left=0.0), None)], {}),
    "unit_one_block": ([(u.keyed_unit(width=50, blocks=1, conv=2, left=0.0), None)], {}),
    "unit_many_blocks": ([(u.keyed_unit(width=66, blocks=22, conv=1, left=0.0), None)], {}),
    "unit_long_filter": ([(u.keyed_unit(width=320, blocks=2, conv=6, left=0.0), None)], {}),
    "dense": ([(u.chunked(), u.dense(limit=0.5))], {}),
    "experts": ([(u.chunked(), u.moe())], {}),
    "one_group": ([(u.chunked(), u.moe(experts=5, top=2, groups=1, keep=1))], {}),
    "groups_of_one": ([(u.chunked(), u.moe(experts=6, top=2, groups=6, keep=3))], {}),
    "all_groups": ([(u.chunked(), u.moe(experts=8, top=3, groups=2, keep=2, scale=1.0))], {}),
    "all_of_the_open": ([(u.chunked(), u.moe(experts=8, top=4, groups=4, keep=2))], {}),
    "one_expert": ([(u.chunked(), u.moe(experts=1, top=1, groups=1, keep=1))], {}),
    "one_bucket": ([(u.chunked(), None)], dict(buckets=1)),
    "large_factors": ([(u.chunked(), None)], dict(buckets=1009, mul_prev=2000003, mul_cur=77777777777, embed_scale=1.0)),
    "loose_caps": ([(u.chunked(), None)], dict(logit_softcap=100.0, residual_mult=1.0, width=100)),
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
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("routes", [(66, 11, 4, 6), (130, 13, 5, 9), (300, 100, 7, 12), (280, 2, 1, 64)], ids=str)
def test_many_experts(xh, act, routes):
    """more experts, and more groups, than a wave has lanes; few tokens and many.  The router reads one dimension only, so that no
    rounding changes the order of its outputs."""
    experts, groups, keep, top = routes
    cfg = u.config([(u.chunked(heads=2, kv_heads=1), u.moe(experts=experts, top=top, groups=groups, keep=keep, ff=16))], width=40)
    w = u.oracle_weights(u.weights(cfg, 2))
    rng = np.random.default_rng(1)
    w["embed"][:, 0], w["bigram"][:, 0] = 5.0 * rng.choice([-1.0, 1.0], cfg["vocab"]), 0.0
    for n in w:
        if n.endswith(".o") or n.endswith(".down"):
            w[n][0] = 0.0
    w["l0.mlp.router"][:] = 0.0
    w["l0.mlp.router"][:, 0] = np.linspace(-1.0, 1.0, experts)[rng.permutation(experts)]
    c = Case(xh, cfg, 2, act, bits={k: u.bf16_bits(v) for k, v in w.items()})
    c.run(0, tokens_of(cfg, 140, 3), [100, 1, 2, 37], "many experts")
    c.free()


def whole_config(**kw):
    return u.config([(u.windowed_delta(), u.dense()), (u.chunked(heads=4, kv_heads=4, dim=16, vdim=16), u.moe()), (u.keyed_unit(), u.moe(experts=9, top=2, groups=3, keep=2)),
                     (u.chunked(heads=4, kv_heads=4, dim=16, vdim=16, kv_from=1, chunk=53), None), (u.windowed_delta(window=65, conv=4), u.moe(top=1)),
                     (u.keyed_unit(heads=3, kv_heads=1, dim=36, rot=36, width=64, blocks=4, conv=3, window=70), None)], **kw)


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
SPAN = 75


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("shape", sorted(SHAPES))
@pytest.mark.parametrize("kind", ["windowed", "keyed", "chunked"])
def test_needle(xh, kind, shape, act):
    """One key decides every later answer that sees it.  It is planted at borders of pages and chunks and elsewhere, and read far away,
    just inside and just outside the window or chunk, in prompts, in portions and by decoded tokens."""
    s = SHAPES[shape]
    scale = 8.0 / s["dim"]
    if kind == "windowed":
        m = u.windowed_delta(vdim=s["dim"], window=SPAN, scale=scale, right=0.0, **s)
    elif kind == "keyed":
        m = u.keyed_unit(rot=s["dim"] // 4 * 2, base=5e5, window=SPAN, scale=scale, right=0.0, **s)
    else:
        m = u.chunked(vdim=s["dim"], chunk=SPAN, scale=scale, softcap=40.0, **s)
    cfg = u.config([(m, None)], width=96)
    bits = u.needle_weights(cfg, 3, key_token=7)
    c = Case(xh, cfg, 0, act, slots=3, max_seq=448, bits=bits)
    for place in (0, 31, 63, 64, 74, 75, 100, 149):
        t = np.random.default_rng(place).integers(8, cfg["vocab"], 260)
        t[place] = 7
        want = c.want(t)
        t2 = t.copy()
        t2[place] = 9
        seen = u.rel_rms(want, c.want(t2))
        last = place // SPAN * SPAN + SPAN - 1 if kind == "chunked" else place + SPAN - 1  # the last position that sees the needle
        assert seen[last + 1] < 1e-9 and (last == place or float(seen[place + 1:last + 1].min()) > 2 * LIMIT["bf16"]), "the needle does not show"
        c.run(0, t, [260], f"{kind} needle at {place}, prompt", want)
        c.run(1, t, [place + 20, 2, 1, 1, 1, 7], f"{kind} needle at {place}, portions", want)
        first = max(last - 2, 1)
        c.run(2, t[:last + 4], [first, 1], f"{kind} needle at {place}, decoded over the edge", want)
        for i in range(3):
            c.model.seq_release(i)
    c.free()


def test_sink_takes_its_weight(xh):
    """sinks far above every score leave little to the values, one far below nothing to itself"""
    cfg = u.config([(u.windowed_delta(heads=3, kv_heads=1, scale=0.05, right=0.0), None)])
    bits = u.weights(cfg, 4)
    bits["l0.mix.left.sink"] = u.bf16_bits(np.array([5.0, -30.0, 2.0]))
    for act in ("f32", "bf16"):
        c = Case(xh, cfg, 0, act, bits=bits)
        t = tokens_of(cfg, 120, 5)
        want = c.want(t)
        c.run(0, t, [120], "prompt", want)
        c.run(1, t, [90, 1], "decoded", want)
        w2 = dict(c.w, **{"l0.mix.left.sink": np.full(3, -1e9)})
        assert u.rel_rms(ref.forward(cfg, w2, t), want).max() > LIMIT["bf16"] * 0.5
        c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_states_remember(xh, act):
    """A recurrence that hardly fades carries the first tokens through hundreds of others, prompt, portions and decoding; what the
    sequence began with shows at its end."""
    for right in (u.windowed_delta(left=0.0, right=1.5), u.keyed_unit(left=0.0, right=1.5)):
        cfg = u.config([(right, None)], residual_mult=1.0)
        w = u.oracle_weights(u.weights(cfg, 5))
        for n in w:
            if n.endswith(".A_log"):
                w[n][:] = -9.0
            if n.endswith(".lam"):
                w[n][:] = -9.0
        c = Case(xh, cfg, 0, act, bits={k: u.bf16_bits(v) for k, v in w.items()})
        t = tokens_of(cfg, 400, 6)
        want = c.want(t)
        t2 = t.copy()
        t2[:12] = tokens_of(cfg, 12, 7)
        assert u.rel_rms(want, c.want(t2))[-1] > 100 * LIMIT["f32"]
        c.run(0, t, [400], "prompt", want)
        c.run(1, t, [130, 2, 65, 1, 1, 100, 64], "portions", want)
        c.run(2, t, [370, 1], "decoded", want)
        c.free()


def test_split_contexts_and_long_portions(xh):
    """long contexts over many parts of the chip, decoded, in short and in long portions"""
    cfg = u.config([(u.chunked(heads=8, kv_heads=2, dim=128, vdim=128, scale=0.2, chunk=1200, softcap=20.0), None),
                    (u.windowed_delta(heads=20, kv_heads=2, dim=64, vdim=128, scale=0.3, window=900), None), (u.keyed_unit(heads=8, kv_heads=1, dim=64, rot=64, window=2000), None)],
                   width=128)
    c = Case(xh, cfg, 12, "bf16", slots=3, max_seq=1600, max_tokens=1600)
    t = tokens_of(cfg, 1500, 6)
    want = c.want(t)
    c.run(0, t, [1100, 1, 1, 2, 5, 16, 1, 17, 56, 99, 1, 1, 1, 200], "long", want)
    for s in (1, 2):
        c.model.step([(s, t[:700 + s], [])])
    got = c.model.step([(1, t[701:702], [0]), (2, t[702:705], [0, 1, 2])])
    c.check(got, want[[701, 702, 703, 704]], "side by side")
    got = c.model.step([(1, t[702:802], [0, 99]), (2, t[705:706], [0])])
    c.check(got, want[[702, 801, 705]], "a long portion beside a token")
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
    c = Case(xh, cfg, 18, act, slots=n, max_seq=64, max_tokens=n * 8)
    prompts = np.stack([tokens_of(cfg, 7, 200 + i) for i in range(n)]).astype(np.int32)
    first, _ = c.model.prefill(prompts, want_logits=True)
    ids = [first] + list(c.model.decode(6, n))
    logits = c.model.logits(n)
    for b in range(n):
        full = np.concatenate([prompts[b], np.stack(ids)[:-1, b]])
        c.check(logits[b:b + 1], c.want(full)[-1:], f"sequence {b}")
    c.free()


def test_slots_that_sit_out(xh):
    cfg = whole_config()
    c = Case(xh, cfg, 14, "f32", slots=3, max_seq=256)
    seqs = [list(tokens_of(cfg, n, 70 + n)) for n in (20, 33, 5)]
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
    # a copy of a slot goes on by itself
    c.model.seq_reorder([2, 0], [1, 1], 0, 0)
    for r in (0, 2):
        seqs[r] = list(seqs[1])
    for r, tok in ((0, 3), (1, 4), (2, 5)):
        c.model.seq_set_next_id(r, tok)
        seqs[r].append(tok)
    c.model.seq_decode([0, 1, 2])
    for r in range(3):
        c.check(c.model.seq_logits(r)[None], c.want(seqs[r])[-1:], f"copied slot {r}")
    c.free()


def test_broken_plans_are_refused(xh):
    layers, _ = u.plan_layers(u.config([(u.chunked(), u.moe()), (u.windowed_delta(), None)]))
    stack = dict(block=2, norm=2)
    attention, left, right = layers
    for change in (dict(heads=5), dict(top=9), dict(top=0), dict(route_groups=5), dict(route_keep=4), dict(window=5), dict(dim=600), dict(out_gate=3), dict(key_values=1),
                   dict(kv_from=1)):
        with pytest.raises(xh.XftHipError):
            xh.Plan(72, 90, [dict(attention, **change)], **stack)
    for bad in ([right], [attention, dict(attention, kv_from=1, vdim=30)], [attention, dict(attention, kv_from=1), dict(attention, kv_from=2)], [left, right, right],
                [left, dict(right, inter=8)], [left, dict(right, decay_rank=4)]):
        with pytest.raises(xh.XftHipError):
            xh.Plan(72, 90, bad, **stack)
    with pytest.raises(xh.XftHipError):  # plain norms do not belong to parallel blocks
        xh.Plan(72, 90, [attention], block=1, norm=2)
    cfg = u.config([(u.windowed_delta(), u.moe()), (u.keyed_unit(), None)])
    bits = u.weights(cfg, 1)
    for name in ("bigram", "l0.mlp.e3.up", "l0.norm2", "l0.mix.left.k.b", "l0.mix.right.dt_bias", "l1.mix.left.k.norm", "l1.mix.right.ri.b"):
        with pytest.raises(xh.XftHipError, match=name.split(".")[-1]):
            u.build_plan(xh, cfg, {k: v for k, v in bits.items() if k != name})


# ---- through the framework's own entry points -----------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dir(tmp_path_factory):
    cfg = whole_config()
    bits = u.steady_weights(cfg, 21)
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
    expect = [greedy(cfg, w, p, 23) for p in prompts]
    out = m.generate(np.array(prompts, np.int32), max_length=40)
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
