"""Plain numpy restatement of the Duvadra decoder, one function per mechanism, for the tests.

Everything runs on whole sequences from position 0, in the dtype of the weights it is given (float64 in the
tests), without a cache, without batching and without sharing any code with the library.  Weights are a
dict name -> array as the model files name them; linear weights are [out, in]."""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def bigram_rows(tokens, b):
    """row of the pair table for every token of a sequence; the first token has one of its own behind the buckets"""
    t = [int(x) for x in tokens]
    return np.array([b["buckets"]] + [(p * b["mul_prev"] + c * b["mul_cur"]) % b["buckets"] for p, c in zip(t, t[1:])])


def embed(tokens, w, e):
    x = w["embed"][np.asarray(tokens)] * e["scale"]
    if e.get("bigram"):
        x = x + w["bigram"][bigram_rows(tokens, e["bigram"])]
    return x


def rotate(x, rot):
    """x [T, heads, n]: pairs (2 i, 2 i + 1) of the first rot.dims entries turned by position * frequency i"""
    n = rot["dims"]
    f = float(rot["base"]) ** (-2.0 * np.arange(n // 2) / n)
    a = np.arange(x.shape[0])[:, None] * f[None, :]
    c, s = np.cos(a)[:, None], np.sin(a)[:, None]
    y = x.copy()
    y[..., 0:n:2] = x[..., 0:n:2] * c - x[..., 1:n:2] * s
    y[..., 1:n:2] = x[..., 1:n:2] * c + x[..., 0:n:2] * s
    return y


def window_mask(T, size):
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & (d < size)


def chunk_mask(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def slopes(H):
    return 2.0 ** (-8.0 * (np.arange(H) + 1) / H)


def attend(q, k, v, mask, scale, sink=None, softcap=None, slope=None):
    """q [T, H, d], k [T, G, d], v [T, G, e], mask [T, T]; sink [H]: one more term of the denominator; softcap bounds the scores;
    slope [H]: what a token of distance costs.  Returns [T, H, e]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    out = np.zeros((T, H, v.shape[-1]), q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if softcap is not None:
            s = softcap * np.tanh(s / softcap)
        if slope is not None:
            s = s - slope[h] * (i - j)
        s = np.where(mask, s, -np.inf)
        m = s.max(-1, keepdims=True)
        if sink is not None:
            m = np.maximum(m, sink[h])
        e = np.exp(s - m)
        den = e.sum(-1, keepdims=True)
        if sink is not None:
            den = den + np.exp(sink[h] - m)
        out[:, h] = (e @ v[:, g]) / den
    return out


def heads(h, w, p, n, bias=False):
    y = h @ w[p].T
    if bias:
        y = y + w[p + ".b"]
    return y.reshape(h.shape[0], n, -1)


def windowed_attention(h, w, p, m):
    """windowed, with a sink, biases and an elementwise output gate, no positions in the scores"""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k, v = heads(h, w, p + "q", H, True), heads(h, w, p + "k", G, True), heads(h, w, p + "v", G, True)
    o = attend(q, k, v, window_mask(T, m["mask"]["size"]), m["scale"], sink=w[p + "sink"])
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def keyed_attention(h, w, p, m, eps):
    """windowed, the projected keys serve as values too; norms over all heads at once, rotation behind them"""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k = h @ w[p + "q"].T, h @ w[p + "k"].T
    v = k.reshape(T, G, -1)
    q = (rms(q, eps) * w[p + "q.norm"]).reshape(T, H, -1)
    k = (rms(k, eps) * w[p + "k.norm"]).reshape(T, G, -1)
    o = attend(rotate(q, m["rot"]), rotate(k, m["rot"]), v, window_mask(T, m["mask"]["size"]), m["scale"])
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def chunked_attention(h, w, p, m, shared):
    """within chunks, capped scores, distances cost, one gate a head; shared: (keys, values) of another layer or None.
    Returns the output and the keys and values it used."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = heads(h, w, p + "q", H)
    kv = shared or (heads(h, w, p + "k", G), heads(h, w, p + "v", G))
    o = attend(q, kv[0], kv[1], chunk_mask(T, m["mask"]["size"]), m["scale"], softcap=m["softcap"], slope=slopes(H))
    return (o * sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, -1) @ w[p + "o"].T, kv


def short_conv(x, taps):
    """Causal convolution over time, one filter a channel: x [T, C], taps [C, n], last tap = the current token."""
    T, n = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for j in range(n):
        back = n - 1 - j
        if back < T:
            y[back:] += x[:T - back] * taps[:, j]
    return y


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, dv], g, beta [T, H]: the state fades, the correction of what the key reads is written, the query
    reads.  Returns [T, H, dv]."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[-1]), q.dtype)
    out = np.zeros_like(v)
    for t in range(T):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hde,hd->he", S, q[t])
    return out


def gated_delta(h, w, p, m, eps):
    T, H, KH, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    part = {n: silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v")}
    q = unit(part["q"].reshape(T, KH, d)) * d ** -0.5
    k = unit(part["k"].reshape(T, KH, d))
    share = np.arange(H) // (H // KH)
    beta = sigmoid(h @ w[p + "b"].T)
    g = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = delta_rule(q[:, share], k[:, share], part["v"].reshape(T, H, dv), g, beta)
    gate = silu(h @ w[p + "g"].T).reshape(T, H, dv)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * dv) @ w[p + "o"].T


def block_gate(u, weight, bias):
    """weight [blocks, n, n], bias [blocks, n]: every part of u through a square matrix of its own"""
    T, B = u.shape[0], weight.shape[0]
    x = u.reshape(T, B, -1)
    return sigmoid(np.stack([x[:, b] @ weight[b].T + bias[b] for b in range(B)], 1)).reshape(T, -1)


def linear_recurrence(a, b):
    """S_t = a_t S_(t-1) + b_t from nothing"""
    out = np.zeros_like(b)
    s = np.zeros(b.shape[-1], b.dtype)
    for t in range(len(b)):
        s = a[t] * s + b[t]
        out[t] = s
    return out


def gated_unit(h, w, p):
    """a real-gated linear recurrent unit behind a short convolution, gated by a second branch"""
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = short_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"]) + w[p + "conv.b"]
    r, i = (block_gate(u, w[p + n], w[p + n + ".b"]) for n in ("ra", "ri"))
    log_a = -8.0 * r * softplus(w[p + "lam"])
    s = linear_recurrence(np.exp(log_a), np.sqrt(-np.expm1(2.0 * log_a)) * i * u)
    return (s * y) @ w[p + "o"].T


def clamped_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(h, w, p, r):
    """[T, experts]: the weight of every expert, zero where it is not chosen"""
    s = sigmoid(h @ w[p + "router"].T)
    T, E = s.shape
    n = r["groups"]["count"]
    parts = s.reshape(T, n, E // n)
    group = np.sort(parts, -1)[:, :, -2:].sum(-1)
    kept = np.argsort(-group, axis=-1, kind="stable")[:, :r["groups"]["keep"]]
    open_ = np.zeros((T, n), bool)
    np.put_along_axis(open_, kept, True, -1)
    choice = np.argsort(-np.where(np.repeat(open_, E // n, 1), s, -np.inf), axis=-1, kind="stable")[:, :r["top"]]
    weight = np.zeros_like(s)
    chosen = np.take_along_axis(s, choice, -1)
    np.put_along_axis(weight, choice, chosen / (chosen.sum(-1, keepdims=True) + 1e-20) * r["scale"], -1)
    return weight


def experts(h, w, p, mlp):
    weight = route(h, w, p, mlp["router"])
    y = np.zeros_like(h)
    for e in range(weight.shape[1]):
        t = np.nonzero(weight[:, e])[0]
        if len(t):
            q = p + "e%d." % e
            y[t] += weight[t, e:e + 1] * ((silu(h[t] @ w[q + "gate"].T) * (h[t] @ w[q + "up"].T)) @ w[q + "down"].T)
    return y


def feed_forward(h, w, p, mlp):
    return clamped_glu(h, w, p, mlp["limit"]) if mlp["kind"] == "dense" else experts(h, w, p, mlp)


def mixer(h, w, cfg, i, kept):
    """kept: keys and values by layer"""
    L, p, eps = cfg["layers"][i], "l%d.mix." % i, cfg["norm"]["eps"]
    m = L["mixer"]
    if L["type"] == "attention":
        j = m.get("kv_from")
        y, kept[i] = chunked_attention(h, w, p, m, None if j is None else kept[j])
        return y
    if L["type"] == "parallel":
        left, right = windowed_attention(h, w, p + "left.", m["left"]), gated_delta(h, w, p + "right.", m["right"], eps)
    else:
        left, right = keyed_attention(h, w, p + "left.", m["left"], eps), gated_unit(h, w, p + "right.")
    return m["left_scale"] * left + m["right_scale"] * right


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of one sequence; streams: a list that receives the residual after every layer."""
    eps, mul = cfg["norm"]["eps"], cfg["residual_mult"]
    x = embed(tokens, w, cfg["embedding"])
    kept = {}
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        x = x + mul * mixer(rms(x, eps) * w[p + "norm1"], w, cfg, i, kept)
        if L.get("mlp"):
            x = x + mul * feed_forward(rms(x, eps) * w[p + "norm2"], w, p + "mlp.", L["mlp"])
        if streams is not None:
            streams.append(x)
    z = (rms(x, eps) * w["final.norm"]) @ w["head"].T
    cap = cfg["logit_softcap"]
    return cap * np.tanh(z / cap)


def param_shapes(cfg):
    """name -> shape of every tensor a configuration needs."""
    W, V, s = cfg["width"], cfg["vocab"], {}
    s["embed"], s["head"], s["final.norm"] = (V, W), (V, W), (W,)
    if cfg["embedding"].get("bigram"):
        s["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)

    def attention(q, m, bias=False, own=True, values=True):
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n, rows, there in (("q", H * d, True), ("k", G * d, own), ("v", G * e, own and values)):
            if there:
                s[q + n] = (rows, W)
                if bias:
                    s[q + n + ".b"] = (rows,)
        s[q + "o"] = (W, H * e)

    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        s[p + "norm1"] = (W,)
        q = p + "mix."
        if L["type"] == "attention":
            attention(q, m, own=m.get("kv_from") is None)
            s[q + "g"] = (m["heads"], W)
        else:
            a, r, l, q = m["left"], m["right"], q + "left.", q + "right."
            attention(l, a, bias=L["type"] == "parallel", values=L["type"] == "parallel")
            s[l + "g"] = (a["heads"] * a["vdim"], W)
            if L["type"] == "parallel":
                s[l + "sink"] = (a["heads"],)
                H, KH, d, dv, n = r["heads"], r["kv_heads"], r["dim"], r["vdim"], r["conv"]
                for t, rows in (("q", KH * d), ("k", KH * d), ("v", H * dv)):
                    s[q + t], s[q + t + ".conv"] = (rows, W), (rows, n)
                s.update({q + "b": (H, W), q + "a": (H, W), q + "A_log": (H,), q + "dt_bias": (H,), q + "norm": (dv,), q + "g": (H * dv, W), q + "o": (W, H * dv)})
            else:
                s[l + "q.norm"], s[l + "k.norm"] = (a["heads"] * a["dim"],), (a["kv_heads"] * a["dim"],)
                R, B = r["width"], r["blocks"]
                n = R // B
                s.update({q + "y": (R, W), q + "y.b": (R,), q + "x": (R, W), q + "x.b": (R,), q + "conv": (R, r["conv"]), q + "conv.b": (R,),
                          q + "ra": (B, n, n), q + "ra.b": (B, n), q + "ri": (B, n, n), q + "ri.b": (B, n), q + "lam": (R,), q + "o": (W, R)})
        f = L.get("mlp")
        if f:
            s[p + "norm2"] = (W,)
            for q, ff in [("", f["ff"])] if f["kind"] == "dense" else [("e%d." % e, f["expert"]["ff"]) for e in range(f["router"]["experts"])]:
                s.update({p + "mlp." + q + "gate": (ff, W), p + "mlp." + q + "up": (ff, W), p + "mlp." + q + "down": (W, ff)})
            if f["kind"] == "moe":
                s[p + "mlp.router"] = (f["router"]["experts"], W)
    return s
