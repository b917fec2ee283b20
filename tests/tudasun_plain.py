"""Plain statement of the Tudasun decoder for the tests: numpy, binary64, one function per mechanism, written out over
tokens and heads.  It shares no code with the product and is as slow as it looks.

A model is (cfg, w): cfg is the dictionary of config.json, w maps tensor names to arrays."""
import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """the model's norm: its weight is stored around zero"""
    return rms(x, eps) * (1.0 + w)


def heads(x, n):
    return x.reshape(x.shape[0], n, -1)


# --- linear attention with a decay per channel ---------------------------------------------------------------
def gated_state(q, k, v, decay, state=None):
    """q, k, decay [T][H][dim], v [T][H][vdim]: S <- diag(decay) S + k v^T, o = S^T q.  Returns (o, S)."""
    T, H, dim = q.shape
    S = np.zeros((H, dim, v.shape[2])) if state is None else state.copy()
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] = decay[t, h][:, None] * S[h] + np.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def gla_decay(z, tau):
    return sigmoid(z) ** (1.0 / tau)


def hgrn2_forget(z, lower):
    return lower + (1.0 - lower) * sigmoid(z)


def gla_mixer(h, m, w, pre, eps, _):
    H = m["heads"]
    q = heads(h @ w[pre + "q"].T, H) * m["dim"] ** -0.5
    k = heads(h @ w[pre + "k"].T, H)
    v = heads(h @ w[pre + "v"].T, H)
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    o, _ = gated_state(q, k, v, heads(gla_decay(z, m["tau"]), H))
    o = (rms(o, eps) * w[pre + "norm"]).reshape(h.shape[0], -1)
    return (o * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def hgrn2_mixer(h, m, w, pre, eps, _):
    H = m["heads"]
    q = heads(silu(h @ w[pre + "q"].T), H)
    v = heads(h @ w[pre + "v"].T, H)
    f = heads(hgrn2_forget(h @ w[pre + "f"].T + w[pre + "f.b"], w[pre + "lower"]), H)
    o, _ = gated_state(q, 1.0 - f, v, f)
    return (rms(o, eps) * w[pre + "norm"]).reshape(h.shape[0], -1) @ w[pre + "o"].T


# --- latent attention ----------------------------------------------------------------------------------------
def rotate(x, pos0, base):
    """the last axis in pairs (2 i, 2 i + 1) turned by position * base^(-2 i / size); axis 0 counts positions"""
    out = np.array(x, np.float64)
    n = x.shape[-1]
    for t in range(x.shape[0]):
        for i in range(n // 2):
            a = (pos0 + t) * base ** (-2.0 * i / n)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * np.cos(a) - v * np.sin(a)
            out[t, ..., 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return out


def softmax_with_sink(s, sink):
    """weights of the scores s; a score without a key, `sink`, takes its share (None: there is none)"""
    m = s.max() if sink is None else max(s.max(), sink)
    e = np.exp(s - m)
    return e / (e.sum() + (0.0 if sink is None else np.exp(sink - m)))


def latent_attention(qn, qr, c, kr, uk, uv, scale, sink, pos0=0):
    """qn [T][H][dim], qr [T][H][rot] (rotated) at positions pos0..; c [N][rank], kr [N][rot] (rotated) of every
    position; uk [H][dim][rank], uv [H][vdim][rank]"""
    T, H, _ = qn.shape
    o = np.zeros((T, H, uv.shape[1]))
    for h in range(H):
        k, v = c @ uk[h].T, c @ uv[h].T
        for t in range(T):
            n = pos0 + t + 1
            s = (k[:n] @ qn[t, h] + kr[:n] @ qr[t, h]) * scale
            o[t, h] = softmax_with_sink(s, None if sink is None else sink[h]) @ v[:n]
    return o


def latent_mixer(h, m, w, pre, eps, shared):
    H, dim, rot, rank = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = heads(h @ w[pre + "q"].T, H)
    base = m["rot"]["base"]
    if m.get("kv_from") is None:
        ckr = h @ w[pre + "dkv"].T
        shared["own"] = rms(ckr[:, :rank], eps) * w[pre + "dkv.norm"], rotate(ckr[:, rank:], 0, base)
        c, kr = shared["own"]
    else:
        c, kr = shared[m["kv_from"]]
    o = latent_attention(q[:, :, :dim], rotate(q[:, :, dim:], 0, base), c, kr, w[pre + "uk"].reshape(H, dim, rank),
                         w[pre + "uv"].reshape(H, m["vdim"], rank), m["scale"], w.get(pre + "sink"))
    return o.reshape(h.shape[0], -1) @ w[pre + "o"].T


MIXERS = {"gla": gla_mixer, "hgrn2": hgrn2_mixer, "latent_attention": latent_mixer}


# --- feed-forward --------------------------------------------------------------------------------------------
def polynorm(z, abce, eps):
    a, b, c, e = abce
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def swiglu(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose(z, correction, top, groups):
    """a token's router logits -> [(output, weight)]: softmax scores, choice by corrected score among the outputs of
    the best groups"""
    s = np.exp(z - z.max())
    s = s / s.sum()
    choice = s + (0.0 if correction is None else correction)
    if groups:
        g = choice.reshape(groups["count"], -1)
        keep = np.argsort(-g.max(axis=1), kind="stable")[:groups["keep"]]
        mask = np.full(g.shape, -np.inf)
        mask[keep] = g[keep]
        choice = mask.reshape(-1)
    ids = np.argsort(-choice, kind="stable")[:top]
    return [(int(i), s[i] / (s[ids].sum() + 1e-20)) for i in ids]


def experts(h, f, w, pre):
    r = f["router"]
    z = h @ w[pre + "router"].T
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for i, weight in choose(z[t], w.get(pre + "correction"), r["top"], r.get("groups")):
            y[t] += weight * (swiglu(h[t:t + 1], w, pre + "e%d." % i)[0] if i < r["experts"] else h[t])
    if f.get("shared"):
        y = y + sigmoid(h @ w[pre + "shared.sg"].T) * swiglu(h, w, pre + "shared.")
    return y


def feed_forward(h, f, w, pre, eps):
    if f["kind"] == "dense":
        return polynorm(h @ w[pre + "up"].T, w[pre + "act"], eps) @ w[pre + "down"].T
    return experts(h, f, w, pre)


# --- layers --------------------------------------------------------------------------------------------------
def side_input(x, e, w, pre, eps):
    g = gelu_tanh(x @ w[pre + "gate"].T) * e
    return rms(g @ w[pre + "proj"].T, eps) * w[pre + "norm"]


def layer(x, tokens, i, cfg, w, latents):
    spec, pre, eps = cfg["layers"][i], "l%d." % i, cfg["norm"]["eps"]
    h = norm(x, w[pre + "norm1"], eps)
    shared = dict(latents)
    y = MIXERS[spec["type"]](h, spec["mixer"], w, pre + "mix.", eps, shared)
    if "own" in shared:
        latents[i] = shared["own"]
    x = x + norm(y * sigmoid(h @ w[pre + "rg1"].T + w[pre + "rg1.b"]), w[pre + "norm1b"], eps)
    if spec.get("mlp"):
        h = norm(x, w[pre + "norm2"], eps)
        y = feed_forward(h, spec["mlp"], w, pre + "mlp.", eps)
        x = x + norm(y * sigmoid(h @ w[pre + "rg2"].T + w[pre + "rg2.b"]), w[pre + "norm2b"], eps)
    if cfg.get("token_side"):
        n = cfg["token_side"]["dim"]
        x = x + side_input(x, w["side.embed"][tokens, i * n:(i + 1) * n], w, pre + "side.", eps)
    return x


def forward(cfg, w, tokens, taps=None):
    """logits [T][vocab] of a whole sequence; `taps` receives the residual stream after every layer"""
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    tokens = np.asarray(tokens)
    x, latents = w["embed"][tokens], {}
    for i in range(len(cfg["layers"])):
        x = layer(x, tokens, i, cfg, w, latents)
        if taps is not None:
            taps.append(x.copy())
    z = norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
    cap = cfg.get("logit_softcap")
    return cap * np.tanh(z / cap) if cap else z


def generate(cfg, w, prompt, n):
    """greedy continuation; also the smallest gap between the best and the second logit met on the way"""
    seq, gap = list(prompt), np.inf
    for _ in range(n):
        z = forward(cfg, w, seq)[-1]
        two = np.sort(z)[-2:]
        gap = min(gap, two[1] - two[0])
        seq.append(int(np.argmax(z)))
    return seq[len(prompt):], gap
