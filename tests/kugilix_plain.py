"""Plain statement of the Kugilix decoder for the tests: numpy, binary64, one function per mechanism, every
loop written out over tokens or heads.  It shares no code with the product and is as slow as it looks.

A model is (cfg, w): cfg is the dictionary of config.json, w maps tensor names to arrays."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def grouped_norm(x, w, groups, eps):
    parts = x.reshape(x.shape[0], groups, -1)
    return rms(parts, eps).reshape(x.shape) * w


def sinusoid(pos, width):
    out = np.zeros(width)
    for e in range(width):
        angle = pos * 10000.0 ** (-2.0 * (e // 2) / width)
        out[e] = np.cos(angle) if e % 2 else np.sin(angle)
    return out


def embed(tokens, table, scale, pos0=0):
    x = np.asarray(table, np.float64)[np.asarray(tokens)] * scale
    for t in range(len(tokens)):
        x[t] += sinusoid(pos0 + t, x.shape[1])
    return x


def causal_conv(h, w, before=None):
    """h + conv(h); `before` holds the inputs ahead of h (zeros when a sequence starts)"""
    T, width = h.shape
    taps = w.shape[1]
    past = np.zeros((taps - 1, width)) if before is None else before
    ext = np.concatenate([past, h], axis=0)
    out = h.copy()
    for t in range(T):
        for j in range(taps):
            out[t] += w[:, j] * ext[t + j]
    return out


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.log1p(np.exp(-np.abs(z))) + np.maximum(z, 0.0)


def xielu(z, p, q):
    pos = softplus(p) * z * z + 0.5 * z
    neg = (0.5 + softplus(q)) * (np.expm1(np.minimum(z, 0.0)) - z) + 0.5 * z
    return np.where(z > 0, pos, neg)


def linear_attention(q, k, v, decay, state=None):
    """q, k [T][heads][dim], v [T][heads][vdim]; S <- decay S + k v^T, o = S^T q.  Returns (o, S)."""
    T, H, _ = q.shape
    S = np.zeros((H, k.shape[2], v.shape[2])) if state is None else state.copy()
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def temperature(pos, coef, every):
    return 1.0 + coef * np.log(np.floor((pos + 1) / every) + 1.0)


def slope(h, H):
    return 2.0 ** (-8.0 * (h + 1) / H)


def window_attention(q, k, v, size, scale, temp=None):
    """q [T][H][dim], k [T][G][dim], v [T][G][vdim], every token of the sequence; softmax over the last `size`
    positions, a bias of slope * distance taken off the scores"""
    T, H, _ = q.shape
    G = k.shape[1]
    o = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = 0 if size is None else max(0, i - size + 1)
        for h in range(H):
            g = h // (H // G)
            qi = q[i, h] * (1.0 if temp is None else temperature(i, *temp))
            s = k[lo:i + 1, g] @ qi * scale - slope(h, H) * (i - np.arange(lo, i + 1))
            p = np.exp(s - s.max())
            o[i, h] = (p / p.sum()) @ v[lo:i + 1, g]
    return o


def heads(x, n):
    return x.reshape(x.shape[0], n, -1)


def attention_mixer(h, m, w, pre, eps):
    H, G = m["heads"], m["kv_heads"]
    q = rms(heads(h @ w[pre + "q"].T, H), eps)
    k = rms(heads(h @ w[pre + "k"].T, G), eps)
    v = heads(h @ w[pre + "v"].T, G)
    temp = (m["q_temp"]["coef"], m["q_temp"]["every"]) if m.get("q_temp") else None
    size = m["mask"]["size"] if m.get("mask") else None
    o = window_attention(q, k, v, size, m["scale"], temp)
    return o.reshape(h.shape[0], -1) @ w[pre + "o"].T


def lightning_mixer(h, m, w, pre, eps):
    H = m["heads"]
    q, k, v = (heads(silu(h @ w[pre + n].T), H) for n in "qkv")
    o, _ = linear_attention(q, k, v, m["decay"])
    o = rms(o.reshape(h.shape[0], -1), eps) * w[pre + "norm"]
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


MIXERS = {"attention": attention_mixer, "lightning": lightning_mixer}


def layer(x, i, cfg, w):
    spec, pre = cfg["layers"][i], "l%d." % i
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    h = causal_conv(grouped_norm(x, w[pre + "norm1"], groups, eps), w[pre + "canon1"])
    y = MIXERS[spec["type"]](h, spec["mixer"], w, pre + "mix.", eps)
    if spec.get("mlp"):
        z = grouped_norm(x, w[pre + "norm2"], groups, eps) @ w[pre + "mlp.up"].T
        p, q = w[pre + "mlp.act"]
        y = y + xielu(z, p, q) @ w[pre + "mlp.down"].T
    return x + y


def layer_runs(cfg):
    """(layer, add the embedding output first) in the order they run"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    runs = [(i, False) for i in range(a)]
    for t in range(times):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, w, tokens, taps=None):
    """logits [T][vocab] of a whole sequence; `taps` receives the residual stream after every layer run"""
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    e = embed(tokens, w["embed"], cfg["embedding"]["scale"])
    x = e.copy()
    for i, again in layer_runs(cfg):
        if again:
            x = x + e
        x = layer(x, i, cfg, w)
        if taps is not None:
            taps.append(x.copy())
    return grouped_norm(x, w["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"]) @ w["head"].T


def generate(cfg, w, prompt, n):
    """greedy continuation; also the smallest gap between the best and the second logit met on the way"""
    seq, gap = list(prompt), np.inf
    for _ in range(n):
        z = forward(cfg, w, seq)[-1]
        two = np.sort(z)[-2:]
        gap = min(gap, two[1] - two[0])
        seq.append(int(np.argmax(z)))
    return seq[len(prompt):], gap
