"""Small random Balenex configurations, their weights, and device plans over them (helpers of the tests)."""
import numpy as np

from oracle import balenex_ref as ref
from plan_util import Case, bf16_bits, bf16_values, oracle_weights, rel_rms  # noqa: F401  (the same for every plan)
import plan_util


def pooled(heads=6, kv_heads=2, dim=20, vdim=28, window=9, pool=3, scale=0.2):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window, pool=pool), scale=scale))


def pair(heads=6, kv_heads=3, dim=20, vdim=12, window=29, keep=7, rot=14, base=3e3, conv=4, scale=0.4, r_heads=3, r_dim=20, r_vdim=28, tau=5.0, rank=6):
    return dict(type="parallel", mixer=dict(
        left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window, keep_first=keep), rot=dict(base=base, dims=rot), conv=conv, scale=scale),
        right=dict(heads=r_heads, dim=r_dim, vdim=r_vdim, tau=tau, _rank=rank)))


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def config(layers, width=72, vocab=90, groups=3, eps=1e-5):
    """layers: (a mixer from above, feed-forward or None)"""
    return dict(architecture="Balenex", width=width, vocab=vocab, norm=dict(eps=eps, groups=groups), layers=[dict(L, mlp=f) for L, f in layers])


def weights(cfg, seed):
    """name -> bf16 bit patterns"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in ref.param_shapes(cfg).items():
        x = rng.standard_normal(shape)
        leaf, parent = (["", ""] + name.split("."))[:-3:-1]
        if "norm" in leaf or leaf == "out":
            x = 1.0 + 0.2 * x
        elif leaf == "b":
            x = rng.uniform(-2.0, 2.0, shape) if parent == "a2" else 0.4 * x
        elif leaf == "conv":
            x *= 0.6
        elif leaf != "embed":
            x *= (2.0 if leaf in ("q", "k", "v") else 1.0) / np.sqrt(shape[-1])
        out[name] = bf16_bits(x)
    for name in out:  # (a read-out near zero would have its sign, and the normed result, decided by rounding)
        if name.endswith("right.k"):
            out[name] = bf16_bits(0.6 * bf16_values(out[name]) + 0.8 * bf16_values(out[name[:-1] + "q"]))
    return out


def needle_weights(cfg, seed, key_token, strength=6.0):
    """Weights under which the token `key_token` has a key that every query scores far above all others, and only attention carries
    anything from token to token: dimension 0 of the residual is the same for all tokens and read by the queries, dimension 1 set for
    key_token alone and read by the keys.  Heads are wide enough for a dimension that is not rotated, or one of the slowest pair."""
    w = oracle_weights(weights(cfg, seed))
    w["embed"][:, 0], w["embed"][:, 1] = strength, 0.0
    w["embed"][key_token, 1] = strength
    for i, L in enumerate(cfg["layers"]):
        one = L["type"] == "attention"
        m, p = (L["mixer"] if one else L["mixer"]["left"]), "l%d.mix." % i + ("" if one else "left.")
        d, rot = m["dim"], (m.get("rot") or {}).get("dims", 0)
        at = rot if rot < d else d // 2 - 1
        for part, heads, source in (("q", m["heads"], 0), ("k", m["kv_heads"], 1)):
            w[p + part] *= 0.2
            for h in range(heads):
                w[p + part][h * d + at] = 0.0
                w[p + part][h * d + at, source] = 4.0
            w[p + part + ".b"][:] = 0.0
            if part == "k":  # (a key of other tokens has a length too)
                w[p + part + ".b"].reshape(heads, d)[:, (at + 1) % d] = 3.0
            if p + part + ".norm" in w:
                w[p + part + ".norm"][:] = 1.0
            if p + part + ".conv" in w:
                w[p + part + ".conv"][:] = 0.0
                w[p + part + ".conv"][:, -1] = 1.0
        if not one:
            w[p + "v.conv"][:] = 0.0
            w[p + "v.conv"][:, -1] = 1.0
            w["l%d.mix.right.out" % i][:] = 0.0
    return {k: bf16_bits(v) for k, v in w.items()}


def plan_layers(cfg):
    """the library's records of a configuration, and the record of every layer"""
    out, record = [], []
    for L in cfg["layers"]:
        m, f, one = L["mixer"], L.get("mlp"), L["type"] == "attention"
        a = m if one else m["left"]
        d = dict(mixer=3, heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"], window=a["mask"]["size"], qkv_bias=1)
        r = None
        if one:
            d.update(qk_norm=3, pool=a["mask"]["pool"], o_bias=1)
        else:
            result = dict(result_norm=1, scaled=1, mix_scale=0.5)
            d.update(qk_norm=1, keep_first=a["mask"]["keep_first"], taps=a["conv"], rot_dim=a["rot"]["dims"], rot_base=a["rot"]["base"], v_rot=1, **result)
            q = m["right"]
            r = dict(mixer=5, heads=q["heads"], dim=q["dim"], vdim=q["vdim"], tau=q["tau"], decay_rank=q["_rank"], beside=1, **result)
        if f:
            d.update(inter=f["ff"], mlp_bias=1)
        record.append(len(out))
        out.append(d)
        if r:
            out.append(r)
    return out, record


STACK = dict(block=0, norm=2)


def build_plan(xh, cfg, bits):
    layers, record = plan_layers(cfg)
    plan = xh.Plan(cfg["width"], cfg["vocab"], layers, eps=cfg["norm"]["eps"], norm_groups=cfg["norm"]["groups"], **STACK)
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


def write_model(path, cfg, bits):
    """config.json + model.safetensors"""
    layers = [dict(L, mixer=dict(L["mixer"], right={k: v for k, v in L["mixer"]["right"].items() if k != "_rank"})) if "right" in L["mixer"] else L for L in cfg["layers"]]
    plan_util.write_model(path, dict(cfg, layers=layers), bits)
