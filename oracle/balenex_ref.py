"""Plain numpy restatement of the Balenex decoder, one function per mechanism, for the tests.

Everything runs on whole sequences from position 0, in the dtype of the weights it is given (float64 in the
tests), without a cache, without batching and without sharing any code with the library.  Weights are a
dict name -> array as the model files name them; linear weights are [out, in]."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def group_rms(x, w, groups, eps):
    """every one of `groups` consecutive parts of a row divided by its own root mean square, the row times w"""
    parts = x.reshape(*x.shape[:-1], groups, -1)
    return rms(parts, eps).reshape(x.shape) * w


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def project(h, w, name):
    """a projection with a bias"""
    return h @ w[name].T + w[name + ".b"]


def short_conv(x, f):
    """x [T, channels], f [channels, taps]: the last tap multiplies the token itself"""
    T, taps = x.shape[0], f.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[j:j + T] * f[:, j] for j in range(taps))


def rotate(x, dims, base, sign=1.0):
    """x [T, heads, n]: entry i of the first `dims` turned together with entry i + dims / 2, by sign * position * base^(-2 i / dims)"""
    half = dims // 2
    a = sign * np.arange(x.shape[0])[:, None] * float(base) ** (-2.0 * np.arange(half) / dims)[None, :]
    c, s = np.cos(a)[:, None], np.sin(a)[:, None]
    y = x.copy()
    y[..., :half] = x[..., :half] * c - x[..., half:dims] * s
    y[..., half:dims] = x[..., half:dims] * c + x[..., :half] * s
    return y


def kept_window_mask(T, size, keep):
    """positions see the last `size` tokens, themselves included, and the sequence's first `keep`"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep))


def window_mask(T, size):
    return kept_window_mask(T, size, 0)


def block_means(x, P):
    """x [T, heads, n] -> means of its whole blocks of P tokens [T // P, heads, n]"""
    n = x.shape[0] // P
    return x[:n * P].reshape(n, P, *x.shape[1:]).mean(1)


def block_mask(T, blocks, P, size):
    """block b is seen once its last token has left the window"""
    i, b = np.arange(T)[:, None], np.arange(blocks)[None, :]
    return b * P + P - 1 <= i - size


def attend(q, k, v, mask, scale):
    """q [T, H, d], k [S, G, d], v [S, G, e], mask [T, S]; query head h reads key / value head h // (H / G)"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.empty((T, H, v.shape[-1]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(mask, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        e = np.exp(s - s.max(-1, keepdims=True))
        out[:, h] = (e / e.sum(-1, keepdims=True)) @ v[:, g]
    return out


def filtered_attention(h, w, p, m, eps):
    """filters on queries, keys and values, head norms, turned values, a window with kept first tokens"""
    T = h.shape[0]
    q, k, v = (short_conv(project(h, w, p + n), w[p + n + ".conv"]).reshape(T, c, -1)
               for n, c in (("q", m["heads"]), ("k", m["kv_heads"]), ("v", m["kv_heads"])))
    rot = m["rot"]
    q = rotate(rms(q, eps) * w[p + "q.norm"], rot["dims"], rot["base"])
    k = rotate(rms(k, eps) * w[p + "k.norm"], rot["dims"], rot["base"])
    v = rotate(v, m["vdim"], rot["base"])
    o = attend(q, k, v, kept_window_mask(T, m["mask"]["size"], m["mask"]["keep_first"]), m["scale"])
    return rotate(o, m["vdim"], rot["base"], -1.0).reshape(T, -1) @ w[p + "o"].T


def decays(h, w, p, tau):
    """of every key channel"""
    return sigmoid((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]) ** (1.0 / tau)


def linear_attention(q, k, v, alpha):
    """q, k, alpha [T, H, d], v [T, H, e]: S = diag(alpha) S + k v^T, read with q behind the write"""
    S, out = np.zeros((q.shape[1], q.shape[2], v.shape[-1])), np.empty_like(v)
    for t in range(len(q)):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def gated_linear(h, w, p, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k, v = ((h @ w[p + n].T).reshape(T, H, -1) for n in "qkv")
    o = linear_attention(q * m["dim"] ** -0.5, k, v, decays(h, w, p, m["tau"]).reshape(T, H, -1))
    o = (rms(o, eps) * w[p + "norm"]).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def pair(left, right, w, p, eps):
    """half the sum of two mixers' results, each normed over the width"""
    return 0.5 * (rms(left, eps) * w[p + "left.out"] + rms(right, eps) * w[p + "right.out"])


def pooled_attention(h, w, p, m, eps):
    """unit heads, a window, and beside its tokens the means of the blocks that lie wholly before it"""
    T, P, size = h.shape[0], m["mask"]["pool"], m["mask"]["size"]
    q, k, v = (project(h, w, p + n).reshape(T, c, -1) for n, c in (("q", m["heads"]), ("k", m["kv_heads"]), ("v", m["kv_heads"])))
    q, k = rms(q, eps), rms(k, eps)
    keys, values = (np.concatenate([x, block_means(x, P)]) for x in (k, v))
    mask = np.concatenate([window_mask(T, size), block_mask(T, T // P, P, size)], 1)
    return project(attend(q, keys, values, mask, m["scale"]).reshape(T, -1), w, p + "o")


def feed_forward(h, w, p):
    hidden = silu(project(h, w, p + "gate")) * project(h, w, p + "up")
    return project(hidden, w, p + "down")


def mixer(h, w, cfg, i):
    L, p, eps = cfg["layers"][i], "l%d.mix." % i, cfg["norm"]["eps"]
    m = L["mixer"]
    if L["type"] == "attention":
        return pooled_attention(h, w, p, m, eps)
    return pair(filtered_attention(h, w, p + "left.", m["left"], eps), gated_linear(h, w, p + "right.", m["right"], eps), w, p, eps)


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of one sequence; streams: a list that receives the residual after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    norm = lambda x, name: group_rms(x, w[name], groups, eps)
    x = w["embed"][np.asarray(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        x = x + norm(mixer(norm(x, p + "norm1"), w, cfg, i), p + "norm1b")
        if L.get("mlp"):
            x = x + norm(feed_forward(norm(x, p + "norm2"), w, p + "mlp."), p + "norm2b")
        if streams is not None:
            streams.append(x)
    return norm(x, "final.norm") @ w["head"].T


def param_shapes(cfg):
    """name -> shape of every tensor a configuration needs; `_rank` of a recurrence: inner width of the decays' projection."""
    W, V, s = cfg["width"], cfg["vocab"], {}
    s["embed"], s["head"], s["final.norm"] = (V, W), (V, W), (W,)
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        s[p + "norm1"], s[p + "norm1b"] = (W,), (W,)
        pairs = L["type"] == "parallel"
        q, a = (p + "mix.left.", m["left"]) if pairs else (p + "mix.", m)
        for n, c, d in (("q", a["heads"], a["dim"]), ("k", a["kv_heads"], a["dim"]), ("v", a["kv_heads"], a["vdim"])):
            s[q + n], s[q + n + ".b"] = (c * d, W), (c * d,)
            if pairs:
                s[q + n + ".conv"] = (c * d, a["conv"])
        s[q + "o"] = (W, a["heads"] * a["vdim"])
        if pairs:
            s[q + "q.norm"], s[q + "k.norm"] = (a["dim"],), (a["dim"],)
            r, q = m["right"], p + "mix.right."
            H, d, e, rank = r["heads"], r["dim"], r["vdim"], r["_rank"]
            s.update({q + "q": (H * d, W), q + "k": (H * d, W), q + "v": (H * e, W), q + "g": (H * e, W), q + "o": (W, H * e), q + "norm": (e,),
                      q + "a1": (rank, W), q + "a2": (H * d, rank), q + "a2.b": (H * d,), p + "mix.left.out": (W,), p + "mix.right.out": (W,)})
        else:
            s[q + "o.b"] = (W,)
        if L.get("mlp"):
            F, q = L["mlp"]["ff"], p + "mlp."
            s[p + "norm2"], s[p + "norm2b"] = (W,), (W,)
            s.update({q + "gate": (F, W), q + "gate.b": (F,), q + "up": (F, W), q + "up.b": (F,), q + "down": (W, F), q + "down.b": (W,)})
    return s
