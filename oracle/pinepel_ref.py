"""Plain numpy restatement of the Pinepel decoder, one function per mechanism, for the tests.

Everything runs on whole sequences from position 0, in the dtype of the weights it is given (float64 in the
tests), without a cache, without batching and without sharing any code with the library.  Weights are a
dict name -> array as the model files name them; linear weights are [out, in]."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm_about_one(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


def rotate(x, base, dims, interleaved, start=0):
    """x [T, heads, n]: the first `dims` entries of every head turned by position * base^(-2 i / dims).
    interleaved: pair i is (2 i, 2 i + 1); else (i, i + dims / 2)."""
    T = x.shape[0]
    half = dims // 2
    f = np.asarray(base, np.float64) ** (-2.0 * np.arange(half) / dims)
    a = (start + np.arange(T))[:, None] * f[None, :]
    c, s = np.cos(a)[:, None, :].astype(x.dtype), np.sin(a)[:, None, :].astype(x.dtype)
    y = x.copy()
    if interleaved:
        u, v = x[..., 0:dims:2], x[..., 1:dims:2]
        y[..., 0:dims:2], y[..., 1:dims:2] = u * c - v * s, v * c + u * s
    else:
        u, v = x[..., :half], x[..., half:dims]
        y[..., :half], y[..., half:dims] = u * c - v * s, v * c + u * s
    return y


def visible(T, window):
    """[T, T] mask: key j is seen from position i.  window 0: all j <= i, else the last `window` of them."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    m = j <= i
    return m & (i - j < window) if window else m


def softmax_with_sink(scores, sink):
    """Rows of scores [..., keys]; sink: one extra logit a row that takes weight but carries no value, or None."""
    mx = scores.max(-1, keepdims=True)
    if sink is not None:
        mx = np.maximum(mx, sink)
    e = np.exp(scores - mx)
    den = e.sum(-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - mx)
    return e / den


def latent_attention(h, w, p, m, eps, interleaved, window, sink):
    """h [T, width]; w: weights; p: prefix of this mixer's names; m: the mixer's sizes."""
    T, H, d, r, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).reshape(T, H, d + r)
    kv = h @ w[p + "dkv"].T
    c = rms(kv[:, :R], eps) * w[p + "dkv.norm"]
    kr = rotate(kv[:, None, R:], m["rot"]["base"], m["rot"]["dims"], interleaved)[:, 0]
    qr = rotate(q[..., d:], m["rot"]["base"], m["rot"]["dims"], interleaved)
    k = (c @ w[p + "uk"].T).reshape(T, H, d)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    s = (np.einsum("ihd,jhd->hij", q[..., :d], k) + np.einsum("ihd,jd->hij", qr, kr)) * m["scale"]
    s = np.where(visible(T, window)[None], s, -np.inf)
    a = softmax_with_sink(s, None if sink is None else sink[:, None, None])
    return np.einsum("hij,jhd->ihd", a, v).reshape(T, H * dv) @ w[p + "o"].T


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
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H]: the state's key rows decay, then the correction of what the
    key reads is written, then the query reads.  Returns [T, H, dv]."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[-1]), q.dtype)
    out = np.zeros_like(v)
    for t in range(T):
        S = S * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hde,hd->he", S, q[t])
    return out


def channel_delta(h, w, p, m, eps):
    T, H, KH, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    part = {n: silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v")}
    q = unit(part["q"].reshape(T, KH, d)) * d ** -0.5
    k = unit(part["k"].reshape(T, KH, d))
    share = np.arange(H) // (H // KH)
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(T, H, d)
    g = np.exp(-np.exp(w[p + "A_log"])[None, :, None] * step)
    o = delta_rule(q[:, share], k[:, share], part["v"].reshape(T, H, dv), g, beta)
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, dv)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * dv) @ w[p + "o"].T


def clamped_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def layer_runs(cfg):
    """(layer, whether the embedding is added in front of it), in running order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def mixer(h, w, cfg, i):
    L, p, eps = cfg["layers"][i], "l%d.mix." % i, cfg["norm"]["eps"]
    m = L["mixer"]
    if L["type"] == "latent_attention":
        return latent_attention(h, w, p, m, eps, True, m["mask"]["size"], None)
    if L["type"] == "latent_attention_2":
        return latent_attention(h, w, p, m, eps, False, 0, w[p + "sink"])
    return channel_delta(h, w, p, m, eps)


def layer(x, w, cfg, i):
    p, eps = "l%d." % i, cfg["norm"]["eps"]
    y = mixer(norm_about_one(x, w[p + "norm1"], eps), w, cfg, i)
    x = x + norm_about_one(y, w[p + "norm1b"], eps) * w[p + "ls1"]
    mlp = cfg["layers"][i].get("mlp")
    if mlp:
        y = clamped_glu(norm_about_one(x, w[p + "norm2"], eps), w, p + "mlp.", mlp["limit"])
        x = x + norm_about_one(y, w[p + "norm2b"], eps) * w[p + "ls2"]
    return x


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of one sequence; streams: a list that receives the residual after every layer run."""
    x0 = w["embed"][np.asarray(tokens)]
    x = x0
    for i, again in layer_runs(cfg):
        if again:
            x = x + x0
        x = layer(x, w, cfg, i)
        if streams is not None:
            streams.append(x)
    return norm_about_one(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T * cfg["logit_scale"]


def param_shapes(cfg):
    """name -> shape of every tensor a configuration needs."""
    W, s = cfg["width"], {}
    s["embed"], s["head"], s["final.norm"] = (cfg["vocab"], W), (cfg["vocab"], W), (W,)
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        for n in ("norm1", "norm1b", "ls1"):
            s[p + n] = (W,)
        q = p + "mix."
        if L["type"] == "channel_delta":
            H, KH, d, dv, n = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            ra, rg = m.get("_a_rank", 16), m.get("_g_rank", 16)
            for t, rows in (("q", KH * d), ("k", KH * d), ("v", H * dv)):
                s[q + t], s[q + t + ".conv"] = (rows, W), (rows, n)
            s.update({q + "b": (H, W), q + "A_log": (H,), q + "norm": (dv,), q + "a1": (ra, W), q + "a2": (H * d, ra),
                      q + "dt_bias": (H * d,), q + "g1": (rg, W), q + "g2": (H * dv, rg), q + "o": (W, H * dv)})
        else:
            H, d, r, dv, R, QR = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            s.update({q + "dq": (QR, W), q + "dq.norm": (QR,), q + "uq": (H * (d + r), QR), q + "dkv": (R + r, W),
                      q + "dkv.norm": (R,), q + "uk": (H * d, R), q + "uv": (H * dv, R), q + "o": (W, H * dv)})
            if L["type"] == "latent_attention_2":
                s[q + "sink"] = (H,)
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            for n in ("norm2", "norm2b", "ls2"):
                s[p + n] = (W,)
            s.update({p + "mlp.gate": (F, W), p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    return s
