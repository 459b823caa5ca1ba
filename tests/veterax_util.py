"""Small random Veterax configurations, their weights, and device plans over them (helpers of the tests)."""
import numpy as np

from oracle import veterax_ref as ref
from plan_util import Case, bf16_bits, bf16_values, oracle_weights, rel_rms, write_model  # noqa: F401  (the same for every plan)


def attention(heads=6, kv_heads=2, dim=20, vdim=28, rot=None, base=5e3, scale=0.5, v_mix=True, scaling=(4.0, 64, 8.0, 1.0)):
    """scaling: factor, original, fast, slow of the context extension, or None"""
    r = dict(base=base, dims=dim if rot is None else rot)
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=r)
    if v_mix is not None:
        m["v_mix"] = v_mix
    return m


def moe(experts=5, identity=2, top=3, ff=24, limit=1.1, shared_ff=40, shared_limit=0.8):
    f = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, identity=identity, top=top))
    if shared_ff:
        f["shared"] = dict(ff=shared_ff, limit=shared_limit)
    return f


def config(layers, width=72, vocab=90, eps=1e-5, side=12):
    """layers: (mixer, feed-forward or None)"""
    c = dict(architecture="Veterax", width=width, vocab=vocab, norm=dict(eps=eps), layers=[dict(type="attention", mixer=m, mlp=f) for m, f in layers])
    if side:
        c["token_side"] = dict(dim=side)
    return c


FEATURES = 4  # leading residual dimensions of steady_weights


def weights(cfg, seed):
    """name -> bf16 bit patterns"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in ref.param_shapes(cfg).items():
        x = rng.standard_normal(shape)
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm") or name == "final.norm":
            x = 1.0 + 0.2 * x
        elif leaf == "alpha":
            x = 0.6 + 0.1 * x
        elif leaf == "b":
            x *= 0.2
        elif leaf == "vmix":
            x = 0.35 + 0.1 * x
        elif leaf == "sink":
            x = 3.0 + x
        elif leaf == "correction":
            x *= 0.3
        elif leaf == "router":
            x *= 2.0 / np.sqrt(shape[-1])
        elif name not in ("embed", "side.embed"):
            x *= (2.5 if leaf == "o" else 1.0) / np.sqrt(shape[-1])  # (what attention finds has to show)
        out[name] = bf16_bits(x)
    return out


def steady_weights(cfg, seed, gap=0.03):
    """Weights whose routing no rounding can turn: the first FEATURES residual dimensions are large, of either sign by token,
    no sublayer but an identity expert writes to them, and the routers read nothing else.  Routers are drawn until every
    combination of signs has its choices at least `gap` apart."""
    rng = np.random.default_rng(seed + 100)
    w = oracle_weights(weights(cfg, seed))
    n = FEATURES
    w["embed"][:, :n] = 5.0 * rng.choice([-1.0, 1.0], (cfg["vocab"], n))
    signs = np.array(np.meshgrid(*[[-1.0, 1.0]] * n)).reshape(n, -1).T
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        w[p + "mix.o"][:n] = 0.0
        if p + "side.norm" in w:
            w[p + "side.norm"][:n] = 0.0
        if not L.get("mlp"):
            continue
        for name in w:
            if name.startswith(p + "mlp.") and name.endswith(".down"):
                w[name][:n] = 0.0
        shape, top = w[p + "mlp.router"].shape, L["mlp"]["router"]["top"]
        h = signs * w[p + "norm2"][:n] + w[p + "norm2.b"][:n]
        for _ in range(20000):
            r = np.zeros(shape)
            r[:, :n] = rng.standard_normal((shape[0], n)) * 0.8
            c = rng.standard_normal(shape[0]) * 0.1
            s = np.sort(ref.softmax(h @ r[:, :n].T) + c, axis=-1)
            if top == shape[0] or (s[:, -top] - s[:, -top - 1]).min() > gap:
                break
        else:
            raise AssertionError("no router with clear choices found")
        w[p + "mlp.router"], w[p + "mlp.correction"] = r, c
    return {k: bf16_bits(v) for k, v in w.items()}


def needle_weights(cfg, seed, key_token, strength=6.0):
    """steady_weights under which the token `key_token` has a key that every query scores far above all others: dimension n of the
    residual is the same for all tokens and read by the queries, dimension n + 1 set for key_token alone and read by the keys.
    The first query / key dimension that is not rotated carries the product, or the slowest pair if all are."""
    w = oracle_weights(steady_weights(cfg, seed))
    ask, key = FEATURES, FEATURES + 1
    w["embed"][:, ask], w["embed"][:, key] = strength, 0.0
    w["embed"][key_token, key] = strength
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], "l%d.mix." % i
        d = m["dim"]
        at = m["rot"]["dims"] if m["rot"]["dims"] < d else d - 2
        for part, heads, source in (("q", m["heads"], ask), ("k", m["kv_heads"], key)):
            for h in range(heads):
                w[p + part][h * d + at] = 0.0
                w[p + part][h * d + at, source] = 3.0 * d ** 0.5
            w[p + part + ".norm"][:] = 1.0
        w["l%d.norm1.b" % i][key] = 0.0
        w[p + "sink"][:] = -4.0
    return {k: bf16_bits(v) for k, v in w.items()}


def plan_layers(cfg):
    """the library's layer descriptions of a configuration"""
    out = []
    for L in cfg["layers"]:
        m, f = L["mixer"], L.get("mlp")
        d = dict(mixer=3, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], rot_dim=m["rot"]["dims"], rot_interleaved=1,
                 rot_base=m["rot"]["base"], scale=m["scale"], has_sink=1, qk_norm=1, v_mix=int(bool(m.get("v_mix"))), window=m.get("_window", 0))
        for k, v in (m["rot"].get("scaling") or {}).items():
            d["rot_" + k] = v
        if f:
            d.update(experts=f["router"]["experts"], identity=f["router"]["identity"], top=f["router"]["top"], expert_inter=f["expert"]["ff"],
                     expert_limit=f["expert"]["limit"], glu_alpha=1.702)
            if f.get("shared"):
                d.update(inter=f["shared"]["ff"], glu_limit=f["shared"]["limit"])
        out.append(d)
    return out


def build_plan(xh, cfg, bits):
    plan = xh.Plan(cfg["width"], cfg["vocab"], plan_layers(cfg), eps=cfg["norm"]["eps"], block=xh.BLOCK_PARALLEL, norm=xh.NORM_DYNAMIC_TANH, tied_head=1,
                   side_dim=(cfg.get("token_side") or {}).get("dim", 0))
    for name, b in bits.items():
        layer, leaf = -1, name
        if name[0] == "l" and name[1].isdigit():
            head, leaf = name.split(".", 1)
            layer = int(head[1:])
        plan.set(layer, leaf, b)
    plan.finish()
    return plan
