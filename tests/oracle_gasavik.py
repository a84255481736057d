"""Float64 numpy restatement of the Gasavik design, one function per mechanism, whole sequence at once with explicit loops over time.

No cache, no state object, no code shared with the package: the recurrences are written as recurrences, the convolutions as sums over earlier positions,
the token shift as a shifted array, attention as a full score matrix with a mask.  `forward(cfg, w, tokens)` returns the logits of every position and the
residual stream after every layer.  `w` maps checkpoint tensor names to float arrays; `cfg` is the dictionary of config.json.
"""
import math

import numpy as np


def rms_unit(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(cfg, w, tokens):
    """token row plus the row of its position, then the norm"""
    x = w["embed"][np.asarray(tokens)] + w["pos"][np.arange(len(tokens))]
    return rms_unit(x, cfg["norm"]["eps"]) * w["embed.norm"]


def token_shift(h, mu):
    """h_t + (h_(t-1) - h_t) * mu with h_(-1) = 0"""
    prev = np.zeros_like(h)
    prev[1:] = h[:-1]
    return h + (prev - h) * mu


def wkv_decay(z, w1, w2, w0):
    """decay per key channel from the mixed input z"""
    return np.exp(-np.exp(np.tanh(z @ w1.T) @ w2.T + w0))


def wkv_recurrence(r, k, v, dec, u):
    """r, k, dec [T, H, d], v [T, H, d], u [H, d]: the read-out sees the past state and, weighted by u, the current token; the state decays row by row"""
    T, H, d = r.shape
    o = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(T):
            kv = np.outer(k[t, h], v[t, h])
            o[t, h] = (S + u[h][:, None] * kv).T @ r[t, h]
            S = dec[t, h][:, None] * S + kv
    return o


def mixer_wkv(m, w, p, h, eps):
    T = h.shape[0]
    H, d = int(m["heads"]), int(m["dim"])
    mixed = {n: token_shift(h, w[p + "mu." + n]) for n in "rkvgw"}
    r, k, v = (np.reshape(mixed[n] @ w[p + n].T, (T, H, d)) for n in "rkv")
    gate = silu(mixed["g"] @ w[p + "g"].T)
    dec = wkv_decay(mixed["w"], w[p + "w1"], w[p + "w2"], w[p + "w0"]).reshape(T, H, d)
    o = wkv_recurrence(r, k, v, dec, w[p + "u"].reshape(H, d))
    o = rms_unit(o, eps).reshape(T, H * d) * w[p + "norm"] * gate
    return o @ w[p + "o"].T


def causal_conv(u, taps_w):
    """u [T, C], taps_w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), nothing before the start"""
    T = u.shape[0]
    taps = taps_w.shape[1]
    y = np.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += taps_w[:, j] * u[: T - back]
    return y


def unit_vector(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_recurrence(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, dv], g, beta [T, H]: decay, correct the value read at k, write, read at q"""
    T, H, d = q.shape
    o = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(T):
            S = g[t, h] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, h])
            S = S + np.outer(k[t, h], u)
            o[t, h] = S.T @ q[t, h]
    return o


def mixer_delta(m, w, p, h, eps):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    share = np.arange(H) // (H // G)
    q = (unit_vector(q.reshape(T, G, d)) * d ** -0.5)[:, share]
    k = unit_vector(k.reshape(T, G, d))[:, share]
    beta = sigmoid(h @ w[p + "b"].T)
    g = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = delta_recurrence(q, k, v.reshape(T, H, dv), g, beta)
    o = rms_unit(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).reshape(T, H, dv)
    return o.reshape(T, H * dv) @ w[p + "o"].T


def visible(i, j, size, keep_first):
    """does position i see position j: the last `size` positions and the first `keep_first` ones (size 0: everything up to i)"""
    return j <= i and (size <= 0 or i - j < size or j < keep_first)


def softmax_attention(q, k, v, scale, kv_heads, size, keep_first):
    T, H, _ = q.shape
    ok = np.array([[visible(i, j, size, keep_first) for j in range(T)] for i in range(T)])
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // kv_heads)
        s = np.where(ok, q[:, h] @ k[:, g].T * scale, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (e / e.sum(axis=1, keepdims=True)) @ v[:, g]
    return out


def mixer_left(m, w, p, h, eps):
    """the attention half of a parallel mixer: biased q / k / v, q / k norm per head, window with kept first tokens, one sigmoid gate per head"""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    mask = m.get("mask") or {}
    q = rms_unit((h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, d), eps) * w[p + "q.norm"]
    k = rms_unit((h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, d), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, dv)
    o = softmax_attention(q, k, v, float(m["scale"]), G, int(mask.get("size", 0)), int(mask.get("keep_first", 0)))
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[p + "o"].T


def lightning_recurrence(q, k, v, decay):
    T, H, d = q.shape
    o = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(T):
            S = decay[h] * S + np.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def mixer_right(m, w, p, h, eps):
    """lightning attention: silu on q, k, v, a fixed decay per head, one norm over all heads, element-wise sigmoid gate"""
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ w[p + n].T).reshape(T, H, d) for n in "qk")
    v = silu(h @ w[p + "v"].T).reshape(T, H, dv)
    o = lightning_recurrence(q, k, v, [float(x) for x in m["decay"]]).reshape(T, H * dv)
    o = rms_unit(o, eps) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def mixer_parallel(m, w, p, h, eps):
    return float(m["left_scale"]) * mixer_left(m["left"], w, p + "left.", h, eps) + float(m["right_scale"]) * mixer_right(m["right"], w, p + "right.", h, eps)


MIXERS = {"wkv": mixer_wkv, "delta": mixer_delta, "parallel": mixer_parallel}


def feed_forward(w, p, h):
    a = silu(h @ w[p + "gate"].T + w[p + "gate.b"]) * (h @ w[p + "up"].T + w[p + "up.b"])
    return a @ w[p + "down"].T + w[p + "down.b"]


def token_side(cfg, w, i, tokens, x, eps):
    """what layer i's own embedding of the token adds to the stream x, before the multiplier"""
    n = int(cfg["token_side"]["dim"])
    e = w["side.embed"][np.asarray(tokens)][:, i * n: (i + 1) * n]
    y = (gelu_tanh(x @ w[f"l{i}.side.gate"].T) * e) @ w[f"l{i}.side.proj"].T
    return rms_unit(y, eps) * w[f"l{i}.side.norm"]


def forward(cfg, w, tokens):
    w = {n: np.asarray(a, np.float64) for n, a in w.items()}
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = embed(cfg, w, tokens)
    states = []
    for i, lc in enumerate(cfg["layers"]):
        h = rms_unit(x, eps) * w[f"l{i}.norm1"]
        d = MIXERS[lc["type"]](lc["mixer"], w, f"l{i}.mix.", h, eps)
        if lc.get("mlp") is not None:
            d = d + feed_forward(w, f"l{i}.mlp.", h)
        x = x + m * d
        if cfg.get("token_side"):
            x = x + m * token_side(cfg, w, i, tokens, x, eps)
        states.append(x.copy())
    return (rms_unit(x, eps) * w["final.norm"]) @ w["head"].T, states
