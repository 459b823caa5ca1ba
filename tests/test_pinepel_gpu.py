"""Layer plans (latent attention, gated delta rule, loops) on the GPU against the plain restatement in
oracle/pinepel_ref.py: every mechanism alone, whole models, portions, batches, page and slot reuse, window and page
borders, long decoding, and generation through AutoModel.  Parity unpinned: the design has no implementation elsewhere."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plan_util as u
from oracle import pinepel_ref as ref

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


ALONE = {
    "windowed": [u.latent(window=13)],
    "windowed_wide_rotation": [u.latent(window=1, heads=1, dim=8, rot=24, vdim=8, kv_rank=24, q_rank=8, base=777.5)],
    "sink": [u.latent()],
    "sink_one_head": [u.latent(heads=1, dim=40, rot=2, vdim=72, kv_rank=72, q_rank=100, scale=1.0)],
    "delta": [u.delta()],
    "delta_equal_heads": [u.delta(heads=2, kv_heads=2, dim=32, vdim=32, conv=3)],
    "delta_long_filter": [u.delta(heads=4, kv_heads=1, dim=8, vdim=40, conv=6, a_rank=1, g_rank=33)],
    "delta_no_filter_memory": [u.delta(heads=3, kv_heads=3, dim=70, vdim=136, conv=1)],
    "delta_wide": [u.delta(heads=2, kv_heads=1, dim=200, vdim=160, conv=2)],
}


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(ALONE))
@pytest.mark.parametrize("mlp", [True, False])
def test_mechanism_alone(xh, name, act, mlp):
    """one layer, prompt and token by token; the residual behind it and the logits"""
    layers = [dict(L) for L in ALONE[name]]
    if not mlp:
        layers[0]["mlp"] = None
    cfg = u.config(layers)
    c = Case(xh, cfg, 11, act)
    t = tokens_of(cfg, 75, 1)
    streams = []
    want = ref.forward(cfg, c.w, t, streams)
    c.model.trace_residual(True)
    got = c.model.step([(0, t, list(range(len(t))))])
    tr = c.model.read_residual()
    assert tr.shape == (1, len(t), cfg["width"])
    c.check(tr[0], streams[0], name + " residual")
    c.check(got, want, name)
    c.model.trace_residual(False)
    c.run(1, t[:20], [1], name + " token by token", want[:20])
    c.free()


def whole_config(**kw):
    return u.config([u.latent(window=37), u.latent(), u.delta(), u.latent(window=70, heads=2, kv_rank=64), u.delta(heads=2, kv_heads=2, dim=32, vdim=24, conv=2)],
                    loop=dict(start=1, stop=4, times=3), **kw)


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_loop_residuals(xh, act):
    """every run of a looped layer, in order; the embedding joins in front of every pass but the first"""
    cfg = whole_config()
    c = Case(xh, cfg, 5, act)
    t = tokens_of(cfg, 40, 2)
    streams = []
    ref.forward(cfg, c.w, t, streams)
    c.model.trace_residual(True)
    c.model.step([(2, t, [])])
    tr = c.model.read_residual()
    assert len(tr) == len(streams) == 1 + 3 * 3 + 1
    for r, s in enumerate(streams):
        c.check(tr[r], s, f"run {r}")
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
@pytest.mark.parametrize("portions", [[300], [1], [2], [3, 2], [64], [63, 1, 65], [31, 33, 2, 1, 120]], ids=str)
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
    live, steps = {}, 0
    made = 0
    while made < 14 or live:
        for s in range(slots):
            pages = sum(-(-len(q["t"]) // 64) for q in live.values())
            if s not in live and made < 14 and rng.random() < 0.7:
                n = int(rng.choice([1, 2, 5, 63, 64, 65, 130, 200]))
                if pages + -(-n // 64) > 9:
                    continue
                t = tokens_of(cfg, n, 100 + made)
                live[s] = dict(t=t, at=0, want=c.want(t), name=made)
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


def test_pool_exhaustion_is_an_error(xh):
    cfg = u.config([u.latent(window=9)])
    c = Case(xh, cfg, 1, "f32", slots=2, max_seq=256, pool=128)
    c.model.step([(0, [1] * 100, [])])
    with pytest.raises(xh.XftHipError, match="exhausted"):
        c.model.step([(1, [1] * 10, [])])
    c.model.seq_release(0)
    c.run(1, tokens_of(cfg, 128, 3), [128], "after the release")
    with pytest.raises(xh.XftHipError):
        c.model.step([(0, [1], [5])])
    with pytest.raises(xh.XftHipError):
        c.model.step([(0, [1], []), (0, [1], [])])
    c.free()


SHAPES = {  # the absorbed kernel's and the expanded kernel's forms: (R, rotated, dim, vdim)
    "wide": dict(heads=2, dim=128, rot=64, vdim=128, kv_rank=512, q_rank=64),
    "half": dict(heads=3, dim=128, rot=32, vdim=128, kv_rank=256, q_rank=40),
    "small": dict(heads=5, dim=64, rot=64, vdim=128, kv_rank=128, q_rank=64),
    "odd": dict(heads=3, dim=100, rot=36, vdim=90, kv_rank=300, q_rank=64),
    "narrow": dict(heads=9, dim=32, rot=32, vdim=32, kv_rank=64, q_rank=72),
    "narrow2": dict(heads=16, dim=64, rot=32, vdim=64, kv_rank=64, q_rank=32),
    "very_wide": dict(heads=1, dim=64, rot=32, vdim=64, kv_rank=640, q_rank=32),
}


@pytest.mark.parametrize("name", sorted(SHAPES))
@pytest.mark.parametrize("window", [None, 50])
def test_needle_bf16(xh, name, window):
    """One key decides every later answer.  It is planted at a page's border and elsewhere, and read just inside and just
    outside the window, far away, in prompts (expanded and absorbed form), in portions and by decoded tokens."""
    cfg = u.config([u.latent(window=window, scale=0.3, **SHAPES[name])], width=96)
    bits = u.needle_weights(cfg, 3, key_token=7)
    c = Case(xh, cfg, 0, "bf16", slots=3, max_seq=448, bits=bits)
    for place in (0, 63, 64, 100, 127):
        t = np.random.default_rng(place).integers(8, cfg["vocab"], 260)
        t[place] = 7
        want, blind = c.want(t), None
        t2 = t.copy()
        t2[place] = 9
        blind = c.want(t2)
        seen = u.rel_rms(want, blind)
        last = place + (window or 400) - 1  # the last position that sees the needle
        assert seen[min(place + 1, 259)] > 0.4 and (last + 1 > 259 or seen[last + 1] < 1e-9), "the needle does not show"
        c.run(0, t, [260], f"{name} needle at {place}, prompt", want)
        c.run(1, t, [place + 20, 2, 1, 1, 1, 7], f"{name} needle at {place}, portions", want)
        if window:
            c.run(2, t[:last + 4], [last - 2, 1], f"{name} needle at {place}, decoded over the edge", want)
        for s in range(3):
            c.model.seq_release(s)
    c.free()


def test_sink_alone_takes_the_weight(xh):
    """a sink far above every score leaves nothing to the values; without it the layer is another one"""
    cfg = u.config([u.latent(scale=0.05)])
    bits = u.weights(cfg, 4)
    bits["l0.mix.sink"] = u.bf16_bits(np.array([5.0, -30.0, 2.0]))
    for act in ("f32", "bf16"):
        c = Case(xh, cfg, 0, act, bits=bits)
        t = tokens_of(cfg, 200, 5)
        want = c.want(t)
        c.run(0, t, [200], "prompt", want)
        c.run(1, t, [190, 1], "decoded", want)
        w2 = dict(c.w, **{"l0.mix.sink": np.full(3, -1e9)})
        assert u.rel_rms(ref.forward(cfg, w2, t), want).min() > LIMIT["bf16"] * 0.5
        c.free()


def test_split_contexts_and_many_heads(xh):
    """long contexts over many parts of the chip, decoded and in short portions"""
    cfg = u.config([u.latent(heads=20, dim=64, rot=64, vdim=64, kv_rank=128, q_rank=64, scale=0.4), u.latent(heads=8, window=333, dim=32, rot=32, vdim=32, kv_rank=256, q_rank=64)],
                   width=128)
    c = Case(xh, cfg, 12, "bf16", slots=3, max_seq=1600, max_tokens=1600)
    t = tokens_of(cfg, 1500, 6)
    want = c.want(t)
    c.run(0, t, [1400, 1, 1, 2, 5, 17, 1, 73], "long", want)
    for s in (1, 2):
        c.model.step([(s, t[:700 + s], [])])
    got = c.model.step([(1, t[701:702], [0]), (2, t[702:705], [0, 1, 2])])
    c.check(got, want[[701, 702, 703, 704]], "side by side")
    c.free()


@pytest.mark.parametrize("act", ["f32", "bf16"])
def test_long_decoding(xh, act):
    """greedy decoding by graph replay: every step's logits row and the chosen ids, then the same steps launched one by one"""
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
        picked = want[29:]
        for i, row in enumerate(picked):
            assert row.max() - row[ids[i, b]] <= 3 * c.limit * want.std(), f"sequence {b}, step {i}"
        c.check(runs[0][1][b:b + 1], want[-1:], f"sequence {b}: logits behind 240 decoded tokens")
    c.free()


def test_slots_that_sit_out_keep_their_state(xh):
    cfg = whole_config()
    c = Case(xh, cfg, 14, "f32", slots=3, max_seq=256)
    seqs = [list(tokens_of(cfg, n, 70 + n)) for n in (20, 33, 5)]
    for s, t in enumerate(seqs):
        c.model.seq_prefill(s, t)
    for rows in ([2], [0, 2], [1], [2, 1], [0], [0, 1, 2]):
        ids = {r: int(c.want(seqs[r])[-1].argmax()) for r in rows}
        for r in rows:
            c.model.seq_set_next_id(r, ids[r])
            seqs[r].append(ids[r])
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


@pytest.mark.parametrize("M", [1, 3, 20, 40, 300])
def test_clamped_gate(xh, M):
    rng = np.random.default_rng(M)
    K, I = 96, 80
    A, W = u.bf16_bits(rng.standard_normal((M, K))), u.bf16_bits(rng.standard_normal((K, 2 * I)) * 0.3)
    w = xh.Weight(xh.W_BF16, K, 2 * I, W, flags=xh.WF_GATEUP)
    a, out = xh.DeviceBuffer.from_numpy(A), xh.DeviceBuffer(M * I * 4)
    import ctypes as C
    xh.check(xh.lib.xfthip_gemm_gateup_clamped(w.h, M, a.ptr, K, out.ptr, I, xh.F32, C.c_float(0.9), C.c_float(1.702), None))
    xh.synchronize()
    gu = u.bf16_values(A) @ u.bf16_values(W)
    g, up = np.minimum(gu[:, :I], 0.9), np.clip(gu[:, I:], -0.9, 0.9)
    np.testing.assert_allclose(out.to_numpy(np.float32, (M, I)), g * ref.sigmoid(1.702 * g) * (up + 1), atol=2e-5)


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
    expect = [greedy(cfg, w, p, 23) for p in prompts]
    out = m.generate(np.array(prompts, np.int32), max_length=40)
    np.testing.assert_array_equal(out, expect)
    # beams: the same number of tokens, the prompt in front; sampling: ids of the vocabulary
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


def test_steps_larger_than_a_pass(xh, tmp_path):
    """a step of more tokens than the device model takes at once runs in several passes: the same logits as in portions"""
    from xfastertransformer_amd.automodel import AutoModel
    cfg = u.config([u.latent(window=50, heads=1), u.delta(heads=2, kv_heads=1)], width=32)
    path = str(tmp_path / "model")
    u.write_model(path, cfg, u.weights(cfg, 30))
    m = AutoModel.from_pretrained(path, "fp32")
    m.set_cache_pool(2 * 8320, 2)
    t = tokens_of(cfg, 8300, 31).tolist()
    places = [0, 8000, 8191, 8192, 8193, 8299]
    ids, a = m.step([(None, t, places), (None, t[:100], [0, 99])])
    m.free_seqs(ids)
    ids, b0 = m.step([(None, t[:4000], [0, 99])])
    _, b1 = m.step([(ids[0], t[4000:], [p - 4000 for p in places[1:]])])
    assert u.rel_rms(a[:6], np.concatenate([b0[:1], b1])).max() < LIMIT["f32"]
    assert u.rel_rms(a[6:], b0).max() < LIMIT["f32"]
    m.free()


def test_unsupported_types_are_refused(xh, model_dir):
    code = ("import sys; sys.path.insert(0, %r)\nfrom xfastertransformer_amd.automodel import AutoModel\n"
            "AutoModel(%r, 'bf16', 'int8')\n" % (ROOT, model_dir[0]))
    p = subprocess.run([sys.executable, "-c", code], capture_output=True, text=True, timeout=100)
    assert p.returncode != 0 and "Unsupported" in p.stdout
    from xfastertransformer_amd.automodel import AutoModel
    with pytest.raises(Exception, match="int8"):
        AutoModel(model_dir[0], "int8")


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
