"""Small random Duvadra configurations, their weights, and device plans over them (helpers of the tests)."""
import numpy as np

from oracle import duvadra_ref as ref
from plan_util import Case, bf16_bits, bf16_values, oracle_weights, rel_rms, write_model  # noqa: F401  (the same for every plan)


def chunked(heads=6, kv_heads=2, dim=20, vdim=28, chunk=37, scale=0.5, softcap=7.0, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=chunk), scale=scale, softcap=softcap)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m)


def windowed_delta(heads=6, kv_heads=3, dim=12, vdim=20, window=29, scale=0.5, r_heads=4, r_kv_heads=2, r_dim=20, r_vdim=12, conv=3, left=0.7, right=1.2):
    return dict(type="parallel", mixer=dict(
        left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), scale=scale), left_scale=left,
        right=dict(heads=r_heads, kv_heads=r_kv_heads, dim=r_dim, vdim=r_vdim, conv=conv), right_scale=right))


def keyed_unit(heads=4, kv_heads=2, dim=24, rot=16, base=3e3, window=33, scale=0.3, width=60, blocks=3, conv=4, left=0.9, right=0.8):
    return dict(type="parallel_2", mixer=dict(
        left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, mask=dict(size=window), scale=scale, rot=dict(base=base, dims=rot)), left_scale=left,
        right=dict(width=width, blocks=blocks, conv=conv), right_scale=right))


def dense(ff=40, limit=1.2):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts=12, top=3, groups=3, keep=2, ff=24, scale=1.9):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, scale=scale, groups=dict(count=groups, keep=keep)))


def config(layers, width=72, vocab=90, eps=1e-5, embed_scale=0.8, buckets=41, mul_prev=13, mul_cur=5, residual_mult=0.6, logit_softcap=3.0):
    """layers: (a mixer from above, feed-forward or None)"""
    return dict(architecture="Duvadra", width=width, vocab=vocab, norm=dict(eps=eps), residual_mult=residual_mult, logit_softcap=logit_softcap,
                embedding=dict(scale=embed_scale, bigram=dict(buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur)),
                layers=[dict(L, mlp=f) for L, f in layers])


FEATURES = 3  # leading residual dimensions of steady_weights
BIASED = ("q", "k", "v", "y", "x", "conv", "ra", "ri")


def weights(cfg, seed):
    """name -> bf16 bit patterns"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in ref.param_shapes(cfg).items():
        x = rng.standard_normal(shape)
        leaf, parent = (["", ""] + name.split("."))[:-3:-1]
        if leaf in ("norm1", "norm2", "norm"):
            x = 1.0 + 0.2 * x
        elif leaf == "b" and parent in BIASED:
            x *= 0.4
        elif leaf == "sink":
            x = 2.5 + x
        elif leaf == "A_log":
            x = rng.uniform(-2.5, 1.0, shape)
        elif leaf == "lam":
            x = rng.uniform(-6.0, 0.0, shape)
        elif leaf == "conv":
            x *= 0.6
        elif leaf == "router":
            x *= 2.0 / np.sqrt(shape[-1])
        elif leaf not in ("embed", "bigram", "dt_bias"):
            x *= (2.5 if leaf == "o" else 1.0) / np.sqrt(shape[-1])  # (what the mixers find has to show)
        out[name] = bf16_bits(x)
    return out


def steady_weights(cfg, seed, gap=0.02):
    """Weights whose routing no rounding can turn: the first FEATURES residual dimensions are large, of either sign by token, no
    sublayer writes to them, and the routers read nothing else.  Routers are drawn until every combination of signs has its choices,
    of groups and of experts, at least `gap` apart at any length of the normed row."""
    rng = np.random.default_rng(seed + 100)
    w = oracle_weights(weights(cfg, seed))
    n = FEATURES
    w["embed"][:, :n] = 5.0 * rng.choice([-1.0, 1.0], (cfg["vocab"], n))
    w["bigram"][:, :n] = 0.0
    signs = np.array(np.meshgrid(*[[-1.0, 1.0]] * n)).reshape(n, -1).T
    for name in w:
        if name.endswith(".o") or (".mlp." in name and name.endswith(".down")):
            w[name][:n] = 0.0
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        if (L.get("mlp") or {}).get("kind") != "moe":
            continue
        r = L["mlp"]["router"]
        groups, keep, top = r["groups"]["count"], r["groups"]["keep"], r["top"]
        shape = w[p + "mlp.router"].shape
        size = shape[0] // groups
        for _ in range(20000):
            m = np.zeros(shape)
            m[:, :n] = rng.standard_normal((shape[0], n)) * 0.6
            least = np.inf
            for length in (0.7, 1.0, 1.5, 2.2):
                s = ref.sigmoid((signs * w[p + "norm2"][:n] * length) @ m[:, :n].T)
                g = np.sort(s.reshape(-1, groups, size), -1)[:, :, -2:].sum(-1)
                if keep < groups:
                    o = np.sort(g, -1)
                    least = min(least, (o[:, -keep] - o[:, -keep - 1]).min())
                kept = np.argsort(-g, -1)[:, :keep]
                mask = np.zeros(g.shape, bool)
                np.put_along_axis(mask, kept, True, -1)
                o = np.sort(np.where(np.repeat(mask, size, 1), s, -1.0), -1)
                if top < keep * size:
                    least = min(least, (o[:, -top] - o[:, -top - 1]).min())
            if least > gap:
                break
        else:
            raise AssertionError("no router with clear choices found")
        w[p + "mlp.router"] = m
    return {k: bf16_bits(v) for k, v in w.items()}


def needle_weights(cfg, seed, key_token, strength=6.0):
    """Weights under which the token `key_token` has a key that every query scores far above all others, and nothing but attention
    carries anything from token to token: dimension 0 of the residual is the same for all tokens and read by the queries, dimension 1
    set for key_token alone and read by the keys.  A query / key dimension that is not rotated carries the product, or one of the
    slowest pair if all are."""
    w = oracle_weights(weights(cfg, seed))
    w["bigram"][:] = 0.0
    w["embed"][:, 0], w["embed"][:, 1] = strength, 0.0
    w["embed"][key_token, 1] = strength
    for i, L in enumerate(cfg["layers"]):
        one = L["type"] == "attention"
        m, p = (L["mixer"] if one else L["mixer"]["left"]), "l%d.mix." % i + ("" if one else "left.")
        d, rot = m["dim"], (m.get("rot") or {}).get("dims", 0)
        at = rot if rot < d else d - 2
        for part, heads, source in (("q", m["heads"], 0), ("k", m["kv_heads"], 1)):
            for h in range(heads):
                w[p + part][h * d + at] = 0.0
                w[p + part][h * d + at, source] = 3.0 * d ** 0.5
            if p + part + ".b" in w:
                w[p + part + ".b"].reshape(heads, d)[:, at] = 0.0
            if p + part + ".norm" in w:
                w[p + part + ".norm"][:] = 1.0
        if p + "sink" in w:
            w[p + "sink"][:] = -4.0
        if not one:
            w["l%d.mix.right.o" % i][:] = 0.0
    return {k: bf16_bits(v) for k, v in w.items()}


def plan_layers(cfg):
    """the library's records of a configuration, and the record of every layer"""
    out, record = [], []
    for L in cfg["layers"]:
        m, f, one, first = L["mixer"], L.get("mlp"), L["type"] == "attention", L["type"] == "parallel"
        a = m if one else m["left"]
        d = dict(mixer=3, heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"])
        d["chunk" if one else "window"] = a["mask"]["size"]
        r = None
        if one:
            d.update(softcap=a["softcap"], distance_bias=1, out_gate=2)
            if a.get("kv_from") is not None:
                d["kv_from"] = record[a["kv_from"]] + 1
        else:
            r = m["right"]
            d.update(out_gate=1, scaled=1, mix_scale=m["left_scale"])
            if first:
                d.update(qkv_bias=1, has_sink=1)
                r = dict(mixer=2, heads=r["heads"], kv_heads=r["kv_heads"], dim=r["dim"], vdim=r["vdim"], taps=r["conv"])
            else:
                d.update(key_values=1, qk_norm=2, rot_dim=a["rot"]["dims"], rot_base=a["rot"]["base"], rot_interleaved=1)
                r = dict(mixer=4, heads=r["blocks"], dim=r["width"] // r["blocks"], vdim=r["width"] // r["blocks"], taps=r["conv"])
            r.update(beside=1, scaled=1, mix_scale=m["right_scale"])
        if f and f["kind"] == "dense":
            d.update(inter=f["ff"], glu_limit=f["limit"], glu_alpha=1.702)
        elif f:
            q = f["router"]
            d.update(experts=q["experts"], top=q["top"], expert_inter=f["expert"]["ff"], router=1, route_groups=q["groups"]["count"],
                     route_keep=q["groups"]["keep"], route_scale=q["scale"])
        record.append(len(out))
        out.append(d)
        if r:
            out.append(r)
    return out, record


def build_plan(xh, cfg, bits):
    layers, record = plan_layers(cfg)
    e = cfg["embedding"]
    plan = xh.Plan(cfg["width"], cfg["vocab"], layers, eps=cfg["norm"]["eps"], block=xh.BLOCK_SERIAL, norm=xh.NORM_RMS, residual_mult=cfg["residual_mult"],
                   embed_scale=e["scale"], logit_softcap=cfg["logit_softcap"], bigram=tuple(e["bigram"][n] for n in ("buckets", "mul_prev", "mul_cur")))
    for name, b in bits.items():
        layer, leaf = -1, name
        if name[0] == "l" and name[1].isdigit():
            head, leaf = name.split(".", 1)
            layer = record[int(head[1:])]
            if leaf.startswith("mix.right."):
                layer, leaf = layer + 1, "mix." + leaf[10:]
            elif leaf.startswith("mix.left."):
                leaf = "mix." + leaf[9:]
        plan.set(layer, leaf, b)
    plan.finish()
    return plan
