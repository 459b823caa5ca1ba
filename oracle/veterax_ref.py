"""Plain numpy restatement of the Veterax decoder, one function per mechanism, for the tests.

Everything runs on whole sequences from position 0, in the dtype of the weights it is given (float64 in the
tests), without a cache, without batching and without sharing any code with the library.  Weights are a
dict name -> array as the model files name them; linear weights are [out, in]."""
import math

import numpy as np


def dynamic_tanh(x, w, p):
    """a squashing in the place of a norm: no statistics of x enter"""
    return np.tanh(w[p + ".alpha"] * x) * w[p] + w[p + ".b"]


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def softmax(z):
    e = np.exp(z - z.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def yarn(dims, base, scaling):
    """(frequency of every pair, factor on cosines and sines): low frequencies are divided by the context's factor, high ones
    stay, a linear ramp over the pair index in between"""
    i = np.arange(dims // 2)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    turns_at = lambda t: dims * math.log(scaling["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns_at(scaling["fast"])), 0), min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate(x, rot, start=0):
    """x [T, heads, n]: pairs (2 i, 2 i + 1) of the first rot.dims entries turned by position * frequency i"""
    n = rot["dims"]
    f, mul = yarn(n, rot["base"], rot.get("scaling"))
    a = (start + np.arange(x.shape[0]))[:, None] * f[None, :]
    c, s = (np.cos(a) * mul)[:, None, :].astype(x.dtype), (np.sin(a) * mul)[:, None, :].astype(x.dtype)
    y = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2], y[..., 1:n:2] = u * c - v * s, v * c + u * s
    return y


def attend(q, k, v, scale, sink, window=0):
    """q [T, H, d], k [T, G, d], v [T, G, e]; every query sees the keys up to its own (window > 0: the last so many of them);
    sink [H]: one more term of the denominator.  Returns [T, H, e]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    out = np.zeros((T, H, v.shape[-1]), q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = np.where((j <= i) & (i - j < (window or T)), (q[:, h] @ k[:, g].T) * scale, -np.inf)
        m = np.maximum(s.max(-1, keepdims=True), sink[h])
        e = np.exp(s - m)
        out[:, h] = (e @ v[:, g]) / (e.sum(-1, keepdims=True) + np.exp(sink[h] - m))
    return out


def attention(h, w, p, m, eps, v_first):
    """returns the mixer's output and this layer's own values (before mixing)"""
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T).reshape(T, H, d), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(T, G, d), eps) * w[p + "k.norm"]
    own = (h @ w[p + "v"].T).reshape(T, G, e)
    v = own
    if v_first is not None:
        lam = w[p + "vmix"]
        v = (1.0 - lam) * own + lam * v_first
    o = attend(rotate(q, m["rot"]), rotate(k, m["rot"]), v, m["scale"], w[p + "sink"], m.get("_window", 0))
    return o.reshape(T, H * e) @ w[p + "o"].T, own


def clamped_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(h, w, p, top):
    """[T, outputs]: the weight of every router output, zero where it is not chosen"""
    s = softmax(h @ w[p + "router"].T)
    choice = np.argsort(-(s + w[p + "correction"]), axis=-1, kind="stable")[:, :top]
    weight = np.zeros_like(s)
    np.put_along_axis(weight, choice, np.take_along_axis(s, choice, -1), -1)
    return weight


def experts(h, w, p, mlp):
    r = mlp["router"]
    weight = route(h, w, p, r["top"])
    y = weight[:, r["experts"]:].sum(-1, keepdims=True) * h  # identity experts
    for e in range(r["experts"]):
        t = np.nonzero(weight[:, e])[0]
        if len(t):
            y[t] += weight[t, e:e + 1] * clamped_glu(h[t], w, p + "e%d." % e, mlp["expert"]["limit"])
    if mlp.get("shared"):
        y = y + clamped_glu(h, w, p + "shared.", mlp["shared"]["limit"])
    return y


def token_side(x, w, p, table, eps):
    """table [T, dim]: this layer's part of the tokens' side embeddings"""
    y = (gelu_tanh(x @ w[p + "side.gate"].T) * table) @ w[p + "side.proj"].T
    return rms(y, eps) * w[p + "side.norm"]


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of one sequence; streams: a list that receives the residual after every layer."""
    tokens = np.asarray(tokens)
    eps = cfg["norm"]["eps"]
    x = w["embed"][tokens]
    v_first = None
    for i, L in enumerate(cfg["layers"]):
        p, mixes = "l%d." % i, bool(L["mixer"].get("v_mix"))
        y, own = attention(dynamic_tanh(x, w, p + "norm1"), w, p + "mix.", L["mixer"], eps, v_first if mixes else None)
        if mixes and v_first is None:
            v_first = own
        if L.get("mlp"):
            y = y + experts(dynamic_tanh(x, w, p + "norm2"), w, p + "mlp.", L["mlp"])
        x = x + y
        if cfg.get("token_side"):
            n = cfg["token_side"]["dim"]
            x = x + token_side(x, w, p, w["side.embed"][tokens][:, i * n:(i + 1) * n], eps)
        if streams is not None:
            streams.append(x)
    return dynamic_tanh(x, w, "final.norm") @ w["embed"].T


def param_shapes(cfg):
    """name -> shape of every tensor a configuration needs."""
    W, s = cfg["width"], {}

    def norm(n):
        s[n], s[n + ".b"], s[n + ".alpha"] = (W,), (W,), ()

    def expert(p, ff):
        s[p + "gate"], s[p + "up"], s[p + "down"] = (ff, W), (ff, W), (W, ff)

    s["embed"] = (cfg["vocab"], W)
    norm("final.norm")
    side = (cfg.get("token_side") or {}).get("dim", 0)
    if side:
        s["side.embed"] = (cfg["vocab"], side * len(cfg["layers"]))
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        norm(p + "norm1")
        q = p + "mix."
        s.update({q + "q": (H * d, W), q + "k": (G * d, W), q + "v": (G * e, W), q + "q.norm": (d,), q + "k.norm": (d,), q + "sink": (H,),
                  q + "o": (W, H * e)})
        if m.get("v_mix"):
            s[q + "vmix"] = ()
        f = L.get("mlp")
        if f:
            norm(p + "norm2")
            r = f["router"]
            for j in range(r["experts"]):
                expert(p + "mlp.e%d." % j, f["expert"]["ff"])
            n = r["experts"] + r["identity"]
            s[p + "mlp.router"], s[p + "mlp.correction"] = (n, W), (n,)
            if f.get("shared"):
                expert(p + "mlp.shared.", f["shared"]["ff"])
        if side:
            s[p + "side.gate"], s[p + "side.proj"], s[p + "side.norm"] = (side, W), (W, side), (W,)
    return s
