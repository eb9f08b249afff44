"""Plain evaluation of block models in double precision, one function per mechanism, straight from the equations.  Slow and
simple; shares nothing with the product.

Weights come as a dict name -> float array (vectors 1-D, matrices [out, in]); `layers` is the configuration's list."""
import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rotate(x, positions, dims, base):
    """x [tokens, heads, size]: adjacent pairs of the first `dims` entries turned by position * base^(-2i/dims)"""
    y = x.copy()
    for i in range(dims // 2):
        a = positions * base ** (-2.0 * i / dims)
        c, s = np.cos(a)[:, None], np.sin(a)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        y[:, :, 2 * i] = u * c - v * s
        y[:, :, 2 * i + 1] = v * c + u * s
    return y


def visible(n, chunk):
    """[query, key]: the keys of the query's own chunk up to itself (chunk 0: all up to itself)"""
    i = np.arange(n)
    m = i[None, :] <= i[:, None]
    if chunk:
        m &= (i[:, None] // chunk) == (i[None, :] // chunk)
    return m


def sink_softmax(scores, mask, sink):
    """rows of weights whose denominator holds exp(sink) as well; sink None: an ordinary softmax"""
    s = np.where(mask, scores, -np.inf)
    top = s.max(axis=1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    den = e.sum(axis=1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - top)
    return e / den


def attention(h, W, p, c, eps, mask=None, with_sink=True):
    n, H, G, d, vd = len(h), c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k = h @ W[p + "q"].T, h @ W[p + "k"].T
    v = (h @ W[p + "v"].T if p + "v" in W else k).reshape(n, G, vd)
    if p + "q.norm" in W:
        q, k = rms_norm(q, W[p + "q.norm"], eps), rms_norm(k, W[p + "k.norm"], eps)
    pos = np.arange(n, dtype=np.float64)
    q = rotate(q.reshape(n, H, d), pos, c["rot"]["dims"], c["rot"]["base"])
    k = rotate(k.reshape(n, G, d), pos, c["rot"]["dims"], c["rot"]["base"])
    m = visible(n, c["mask"]["size"]) if mask is None else mask
    out = np.zeros((n, H, vd))
    for head in range(H):
        g = head // (H // G)
        sink = W[p + "sink"][head] if with_sink and p + "sink" in W else None
        out[:, head] = sink_softmax(q[:, head] @ k[:, g].T * c["scale"], m, sink) @ v[:, g]
    return out.reshape(n, H * vd) @ W[p + "o"].T


def causal_conv(x, w):
    """per channel, last column of w on the current token, nothing before the start; then silu"""
    n, taps = len(x), w.shape[1]
    y = np.zeros_like(x)
    for t in range(n):
        for j in range(taps):
            if t - j >= 0:
                y[t] += w[:, taps - 1 - j] * x[t - j]
    return silu(y)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_recurrence(q, k, v, beta, g):
    """q, k, g [n, heads, dim], v [n, heads, vdim], beta [n, heads] -> read-outs [n, heads, vdim]"""
    n, H, d = k.shape
    out = np.zeros_like(v)
    for head in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(n):
            S = g[t, head][:, None] * S
            u = beta[t, head] * (v[t, head] - S.T @ k[t, head])
            S = S + np.outer(k[t, head], u)
            out[t, head] = S.T @ q[t, head]
    return out


def delta_rule(h, W, p, c, eps):
    n, H, G, d, vd = len(h), c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = causal_conv(h @ W[p + "q"].T, W[p + "q.conv"]).reshape(n, G, d)
    k = causal_conv(h @ W[p + "k"].T, W[p + "k.conv"]).reshape(n, G, d)
    v = causal_conv(h @ W[p + "v"].T, W[p + "v.conv"]).reshape(n, H, vd)
    q, k = unit(q) / np.sqrt(d), unit(k)
    q, k = np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1)
    beta = sigmoid(h @ W[p + "b"].T)
    raw = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    g = np.exp(-np.exp(W[p + "A_log"])[None, :, None] * softplus(raw).reshape(n, H, d))
    o = delta_recurrence(q, k, v, beta, g)
    gate = sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).reshape(n, H, vd)
    return (rms_norm(o, W[p + "norm"], eps) * gate).reshape(n, H * vd) @ W[p + "o"].T


def choose_experts(z, top):
    """indices of the `top` largest scores, the lower index first on equal ones"""
    return np.argsort(-z, axis=-1, kind="stable")[..., :top]


def mixture(h, W, p, top):
    z = h @ W[p + "router"].T
    out = np.zeros_like(h)
    for t, picks in enumerate(choose_experts(z, top)):
        for e in picks:
            x = sigmoid(z[t, e]) * h[t]
            out[t] += W[f"{p}e{e}.down"] @ (silu(W[f"{p}e{e}.gate"] @ x) * (W[f"{p}e{e}.up"] @ x))
    return out


def forward(tokens, W, cfg, **attention_options):
    """logits [n, vocab] and the residual stream behind every mixer and every layer"""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)].astype(np.float64)
    behind_mixer, behind_layer = [], []
    for i, layer in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", layer["mixer"]
        h = rms_norm(x, W[p + "norm1"], eps)
        y = 0.0
        if mix["left"]:
            y = y + mix["left_scale"] * attention(h, W, p + "mix.left.", mix["left"], eps, **attention_options)
        if mix["right"]:
            y = y + mix["right_scale"] * delta_rule(h, W, p + "mix.right.", mix["right"], eps)
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        behind_mixer.append(x)
        if layer["mlp"]:
            y = mixture(rms_norm(x, W[p + "norm2"], eps), W, p + "mlp.", layer["mlp"]["router"]["top"])
            x = x + rms_norm(y, W[p + "norm2b"], eps)
        behind_layer.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T, behind_mixer, behind_layer


def greedy(tokens, count, W, cfg):
    seq = list(tokens)
    for _ in range(count):
        seq.append(int(np.argmax(forward(seq, W, cfg)[0][-1])))
    return seq[len(tokens):]
