"""Small random Pinepel configurations, their weights, and device models over them (helpers of the layer-plan tests)."""
import json
import os
import struct

import numpy as np

from oracle import pinepel_ref as ref


def latent(heads=3, dim=24, rot=8, vdim=20, kv_rank=40, q_rank=28, scale=0.2, base=1e4, window=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, rot=dict(base=base, dims=rot))
    if window is not None:
        m["mask"] = dict(size=window)
    return dict(type="latent_attention_2" if window is None else "latent_attention", mixer=m)


def delta(heads=6, kv_heads=2, dim=20, vdim=12, conv=4, a_rank=6, g_rank=10):
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, _a_rank=a_rank, _g_rank=g_rank))


def config(layers, width=72, vocab=90, ff=56, limit=1.3, loop=None, eps=1e-5, logit_scale=1.7):
    out = []
    for i, L in enumerate(layers):
        L = dict(L)
        if "mlp" not in L:
            L["mlp"] = dict(kind="dense", ff=ff + 8 * i, limit=limit)
        out.append(L)
    return dict(architecture="Pinepel", width=width, vocab=vocab, norm=dict(eps=eps), logit_scale=logit_scale, layers=out, loop=loop)


def bf16_bits(x):
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits):
    return (bits.astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def weights(cfg, seed):
    """name -> bf16 bit patterns"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in ref.param_shapes(cfg).items():
        x = rng.standard_normal(shape)
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm1b", "norm2b") or name == "final.norm":
            x *= 0.2
        elif leaf in ("ls1", "ls2") or leaf == "norm":
            x = 1.0 + 0.2 * x
        elif leaf == "conv":
            x *= 0.6
        elif leaf == "A_log":
            x = rng.uniform(-2.0, 1.5, shape)
        elif leaf == "sink":
            x = 2.0 + x
        elif leaf not in ("embed", "dt_bias"):
            x /= np.sqrt(shape[-1])
        out[name] = bf16_bits(x)
    return out


def oracle_weights(bits):
    return {k: bf16_values(v) for k, v in bits.items()}


def plan_layers(cfg):
    """the library's layer descriptions of a configuration"""
    out = []
    for L in cfg["layers"]:
        m = L["mixer"]
        d = dict(heads=m["heads"], dim=m["dim"], vdim=m["vdim"])
        if L["type"] == "channel_delta":
            d.update(mixer=2, kv_heads=m["kv_heads"], taps=m["conv"], decay_rank=m["_a_rank"], gate_rank=m["_g_rank"])
        else:
            windowed = L["type"] == "latent_attention"
            d.update(mixer=1, rot_dim=m["rot_dim"], kv_rank=m["kv_rank"], q_rank=m["q_rank"], scale=m["scale"], rot_base=m["rot"]["base"],
                     rot_interleaved=int(windowed), window=m["mask"]["size"] if windowed else 0, has_sink=int(not windowed))
        if L.get("mlp"):
            d.update(inter=L["mlp"]["ff"], glu_limit=L["mlp"]["limit"], glu_alpha=1.702)
        out.append(d)
    return out


def build_plan(xh, cfg, bits):
    loop = cfg.get("loop") or dict(start=0, stop=0, times=1)
    plan = xh.Plan(cfg["width"], cfg["vocab"], plan_layers(cfg), (loop["start"], loop["stop"], loop["times"]), cfg["norm"]["eps"], cfg["logit_scale"])
    for name, b in bits.items():
        layer, leaf = -1, name
        if name[0] == "l" and name[1].isdigit():
            head, leaf = name.split(".", 1)
            layer = int(head[1:])
        plan.set(layer, leaf, b)
    plan.finish()
    return plan


def write_model(path, cfg, bits):
    """config.json + model.safetensors"""
    os.makedirs(path, exist_ok=True)
    c = json.loads(json.dumps(cfg))
    for L in c["layers"]:
        for k in [k for k in L["mixer"] if k.startswith("_")]:
            del L["mixer"][k]
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(c, f)
    header, at, blobs = {}, 0, []
    for name, b in bits.items():
        raw = np.ascontiguousarray(b, "<u2").tobytes()
        header[name] = dict(dtype="BF16", shape=list(b.shape), data_offsets=[at, at + len(raw)])
        at += len(raw)
        blobs.append(raw)
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))


def rel_rms(got, want):
    """root mean square difference of every row over the rows' overall spread"""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.sqrt(((got - want) ** 2).mean(-1)) / max(want.std(), 1e-9)


class Case:
    """A device model over a plan, held against an oracle: forward(weights, tokens) -> logits."""

    def __init__(self, xh, plan, w, forward, act, limit, slots=4, max_seq=512, max_tokens=None, pool=0):
        self.w, self.plan, self.limit, self.forward = w, plan, limit, forward
        self.model = xh.PlanModel(plan, xh.F32 if act == "f32" else xh.BF16, slots, max_seq, max_tokens or max_seq, pool)

    def want(self, tokens):
        return self.forward(self.w, tokens)

    def check(self, got, want, what, rows=None):
        err = rel_rms(got, want if rows is None else want[rows])
        assert err.max() < self.limit, f"{what}: row {int(err.argmax())} of {len(err)} differs by {err.max():.2e} (limit {self.limit})"

    def run(self, slot, tokens, portions, what, want=None):
        """the sequence in portions of the given sizes (the last size repeats), all logits checked"""
        want = self.want(tokens) if want is None else want
        at, i = 0, 0
        while at < len(tokens):
            n = min(portions[min(i, len(portions) - 1)], len(tokens) - at)
            got = self.model.step([(slot, tokens[at:at + n], list(range(n)))])
            self.check(got, want[at:at + n], f"{what}, portion {i} at {at}")
            at, i = at + n, i + 1

    def free(self):
        self.model.free()
        self.plan.free()


# ---- needles: a prompt in which one key decides the answer ------------------------------------------------------------
def needle_weights(cfg, seed, key_token, strength=6.0):
    """Weights under which the token `key_token` has a key that every query of the latent layers scores far above all
    others: the tokens' embeddings share a direction that the queries read, key_token alone has the one the keys read."""
    bits = weights(cfg, seed)
    w = oracle_weights(bits)
    rng = np.random.default_rng(seed + 1)
    W = cfg["width"]
    ask, key = np.zeros(W), np.zeros(W)
    ask[0], key[1] = 1.0, 1.0
    e = w["embed"] * 0.5
    e[:, 0], e[:, 1] = strength, 0.0
    e[key_token, 1] = strength
    w["embed"] = e
    for i, L in enumerate(cfg["layers"]):
        if L["type"] == "channel_delta":
            continue
        m, p = L["mixer"], "l%d.mix." % i
        d, r, H = m["dim"], m["rot_dim"], m["heads"]
        # query latent 0 carries `ask`, key latent 0 carries `key`; every head multiplies the two
        for t in ("dq", "dkv"):
            w[p + t][0] = 0.0
        w[p + "dq"][0, 0], w[p + "dkv"][0, 1] = 4.0, 4.0
        for h in range(H):
            w[p + "uq"][h * (d + r)] = 0.0
            w[p + "uq"][h * (d + r), 0] = 3.0
            w[p + "uk"][h * d] = 0.0
            w[p + "uk"][h * d, 0] = 3.0
        if p + "sink" in w:
            w[p + "sink"][:] = -4.0
    del rng, ask, key
    return {k: bf16_bits(v) for k, v in w.items()}
