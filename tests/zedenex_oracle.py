"""Plain evaluation of Zedenex models in double precision, one function per mechanism, straight from the equations.  Slow and
simple; shares nothing with the product.

Weights come as a dict name -> float array (scalars 0-D, vectors 1-D, matrices [out, in]); `cfg` is the configuration."""
import numpy as np

from block_oracle import attention, delta_rule, mixture, rms_norm, rotate, silu, sink_softmax, softplus


def dynamic_tanh(x, alpha, w, b):
    return np.tanh(alpha * x) * w + b


def embedding(tokens, W, c):
    """scaled table rows plus a row of the bigram table, chosen by the token and the one before it; a sequence's first token
    takes the bigram table's last row"""
    tokens = [int(t) for t in tokens]
    x = W["embed"][tokens] * c["scale"]
    g = c.get("bigram")
    if g:
        rows = [g["buckets"]] + [(a * g["mul_prev"] + b * g["mul_cur"]) % g["buckets"] for a, b in zip(tokens, tokens[1:])]
        x = x + W["bigram"][rows]
    return x


def gather_streams(x, weights):
    """x [streams, tokens, width] -> the sublayer's input"""
    return np.tensordot(weights, x, 1)


def spread_streams(x, mix, out, y):
    """all streams from the old ones (mix[from, to]) and the sublayer's output"""
    return np.einsum("ft,fnd->tnd", mix, x) + out[:, None, None] * y


def run_order(cfg):
    """layer of every pass"""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def latent_attention(h, W, p, c, eps, mask=None, with_sink=True):
    n, H, d, r, vd, kr = len(h), c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    q = (rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T).reshape(n, H, d + r)
    both = h @ W[p + "dkv"].T
    latent = rms_norm(both[:, :kr], W[p + "dkv.norm"], eps)
    pos = np.arange(n, dtype=np.float64)
    kr_rot = rotate(both[:, None, kr:], pos, c["rot"]["dims"], c["rot"]["base"])[:, 0]
    q_rot = rotate(q[:, :, d:], pos, c["rot"]["dims"], c["rot"]["base"])
    k = (latent @ W[p + "uk"].T).reshape(n, H, d)
    v = (latent @ W[p + "uv"].T).reshape(n, H, vd)
    m = np.tril(np.ones((n, n), bool)) if mask is None else mask
    out = np.zeros((n, H, vd))
    for head in range(H):
        s = (q[:, head, :d] @ k[:, head].T + q_rot[:, head] @ kr_rot.T) * c["scale"]
        out[:, head] = sink_softmax(s, m, W[p + "sink"][head] if with_sink and p + "sink" in W else None) @ v[:, head]
    return out.reshape(n, H * vd) @ W[p + "o"].T


def biased_causal_conv(x, w, b):
    """per channel, last column of w on the current token, nothing before the start; then silu"""
    n, taps = len(x), w.shape[1]
    y = np.tile(b, (n, 1))
    for j in range(taps):
        y[j:] += w[:, taps - 1 - j] * x[:n - j]
    return silu(y)


def state_space(x, B, C, dt, a_log, D):
    """x [n, heads, vdim], B and C [n, heads, state], dt [n, heads] -> read-outs [n, heads, vdim]"""
    n, H, vd = x.shape
    out = np.zeros_like(x)
    for head in range(H):
        S = np.zeros((B.shape[2], vd))
        for t in range(n):
            S = np.exp(-np.exp(a_log[head]) * dt[t, head]) * S + dt[t, head] * np.outer(B[t, head], x[t, head])
            out[t, head] = S.T @ C[t, head] + D[head] * x[t, head]
    return out


def grouped_rms_norm(x, groups, w, eps):
    parts = x.reshape(len(x), groups, -1)
    return (parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)).reshape(x.shape) * w


def mamba2(h, W, p, c, eps):
    n, H, G, N, vd = len(h), c["heads"], c["groups"], c["state"], c["vdim"]
    inner = H * vd
    z, xbc, dt = np.split(h @ W[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = biased_causal_conv(xbc, W[p + "conv"], W[p + "conv.b"])
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    B, C = (np.repeat(a.reshape(n, G, N), H // G, axis=1) for a in (B, C))
    y = state_space(x.reshape(n, H, vd), B, C, softplus(dt + W[p + "dt_bias"]), W[p + "A_log"], W[p + "D"])
    return grouped_rms_norm(y.reshape(n, inner) * silu(z), c["norm_groups"], W[p + "norm"], eps) @ W[p + "o"].T


def dense(h, W, p, act="relu"):
    g = h @ W[p + "gate"].T
    return ((np.maximum(g, 0.0) if act == "relu" else silu(g)) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def sublayers(layer, p, W, eps, **attention_options):
    """what a layer does, one function per sublayer: the mixer, and the feed-forward if it has one"""
    m = layer["mixer"]
    if layer["type"] == "latent_attention":
        yield lambda h: latent_attention(h, W, p + "mix.", m, eps, **attention_options)
    elif layer["type"] == "mamba2":
        yield lambda h: mamba2(h, W, p + "mix.", m, eps)
    else:
        yield lambda h: m["left_scale"] * attention(h, W, p + "mix.left.", m["left"], eps) + m["right_scale"] * delta_rule(h, W, p + "mix.right.", m["right"], eps)
    mlp = layer["mlp"]
    if mlp and mlp["kind"] == "moe":
        yield lambda h: mixture(h, W, p + "mlp.", mlp["router"]["top"])
    elif mlp:
        yield lambda h: dense(h, W, p + "mlp.", mlp.get("act", "relu"))


def norm(x, W, name, eps):
    """by what the weights hold: a tanh norm or an RMS norm"""
    return dynamic_tanh(x, W[name + ".alpha"], W[name], W[name + ".b"]) if name + ".alpha" in W else rms_norm(x, W[name], eps)


def forward(tokens, W, cfg, **attention_options):
    """logits [n, vocab]; the sum of the streams behind every mixer and behind every layer, pass by pass.  Without streams: one
    residual, and a norm on each sublayer's output."""
    eps = cfg["norm"]["eps"]
    x = np.stack([embedding(tokens, W, cfg["embedding"])] * max(1, cfg["streams"]))
    behind = [[], []]
    for i in run_order(cfg):
        p = f"l{i}."
        for q, f in enumerate(sublayers(cfg["layers"][i], p, W, eps, **attention_options), 1):
            hc, n = f"{p}hc{q}.", f"{p}norm{q}"
            if cfg["streams"]:
                x = spread_streams(x, W[hc + "mix"], W[hc + "out"], f(norm(gather_streams(x, W[hc + "in"]), W, n, eps)))
            else:
                x = x + rms_norm(f(norm(x[0], W, n, eps)), W[n + "b"], eps)
            if q == 1:
                behind[0].append(x.sum(0))
        behind[1].append(x.sum(0))
    return norm(x.sum(0), W, "final.norm", eps) @ W["head" if "head" in W else "embed"].T, *behind


def greedy(tokens, count, W, cfg):
    seq = list(tokens)
    for _ in range(count):
        seq.append(int(np.argmax(forward(seq, W, cfg)[0][-1])))
    return seq[len(tokens):]
