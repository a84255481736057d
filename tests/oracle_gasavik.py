"""Float64 numpy restatement of the Gasavik design, one function per mechanism, whole sequence at once with explicit loops over time.

No cache, no state object, no code shared with the package: the recurrences are written as recurrences, the convolutions as sums over earlier positions,
the token shift as a shifted array, attention as a full score matrix with a mask.  `forward(cfg, w, tokens)` returns the logits of every position and the
residual stream after every layer.  `w` maps checkpoint tensor names to float arrays; `cfg` is the dictionary of config.json.
"""
import json
import math
import os
import struct

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


# ------------------------------------------------------------------------------------------------ configurations and weights of the tests
def wkv(heads, dim, rank=4):
    """rank: only the checkpoint's tensors show it"""
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "rank": rank}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def parallel(heads, kv_heads, dim, vdim, size, keep_first, lt_heads, lt_dim, lt_vdim, scale=None, left_scale=0.7, right_scale=1.3, decay=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}
    if size:
        left["mask"] = {"size": size, "keep_first": keep_first}
    dec = [1.0 - 2.0 ** (-1.0 - 7.0 * (h + 1) / lt_heads) for h in range(lt_heads)] if decay is None else list(decay)
    return {"type": "parallel", "mixer": {"left": left, "left_scale": left_scale, "right": {"heads": lt_heads, "dim": lt_dim, "vdim": lt_vdim, "decay": dec}, "right_scale": right_scale}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def make_config(width, vocab, layers, eps=1e-5, residual_mult=0.6, side=5, positions=1536):
    cfg = {"architecture": "Gasavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": residual_mult, "max_positions": positions,
           "layers": [{k: v for k, v in l.items() if k != "rank"} for l in layers], "_ranks": [l.get("rank", 0) for l in layers]}
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg


def random_weights(cfg, seed):
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}

    def mat(name, *shape, gain=1.0):
        out[name] = (rng.standard_normal(shape) * gain / math.sqrt(shape[-1])).astype(np.float32)

    def vec(name, *shape, mid=0.0, amp=0.2):
        out[name] = (mid + amp * rng.standard_normal(shape)).astype(np.float32)
    vec("embed", V, W, amp=0.8); vec("pos", cfg["max_positions"], W, amp=0.4)
    vec("embed.norm", W, mid=1.0); vec("final.norm", W, mid=1.0)
    mat("head", V, W)
    ns = int((cfg.get("token_side") or {}).get("dim", 0))
    if ns:
        vec("side.embed", V, ns * len(cfg["layers"]), amp=1.0)
    for i, lc in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lc["mixer"], lc.get("mlp")
        q = p + "mix."
        vec(p + "norm1", W, mid=1.0)
        if lc["type"] == "wkv":
            H, d, rank = m["heads"], m["dim"], cfg["_ranks"][i]
            for n in "rkvgw":
                out[q + "mu." + n] = rng.uniform(0.0, 1.0, W).astype(np.float32)
            for n in "rkvg":
                mat(q + n, H * d, W, gain=1.2)
            mat(q + "w1", rank, W, gain=2.0); mat(q + "w2", H * d, rank); vec(q + "w0", H * d, mid=-2.0, amp=1.5); vec(q + "u", H, d, amp=0.8)
            vec(q + "norm", H * d, mid=1.0); mat(q + "o", W, H * d)
        elif lc["type"] == "delta":
            H, G, d, dv, taps = (m[k] for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                mat(q + n, rows, W, gain=1.5)
                out[q + n + ".conv"] = (rng.standard_normal((rows, taps)) * 0.6).astype(np.float32)
            mat(q + "b", H, W, gain=2.0); mat(q + "a", H, W); vec(q + "A_log", H, mid=-1.0, amp=1.0); vec(q + "dt_bias", H, mid=-1.0, amp=1.0)
            vec(q + "norm", dv, mid=1.0); mat(q + "g", H * dv, W); mat(q + "o", W, H * dv)
        else:
            a, b = m["left"], m["right"]
            H, G, d, dv = (a[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                mat(q + "left." + n, rows, W, gain=1.5); vec(q + "left." + n + ".b", rows)
            vec(q + "left.q.norm", d, mid=1.5); vec(q + "left.k.norm", d, mid=1.5)
            mat(q + "left.g", H, W); mat(q + "left.o", W, H * dv)
            H, d, dv = (b[k] for k in ("heads", "dim", "vdim"))
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                mat(q + "right." + n, rows, W, gain=1.3)
            vec(q + "right.norm", H * dv, mid=1.0); mat(q + "right.o", W, H * dv)
        if f is not None:
            for n, shape in (("gate", (f["ff"], W)), ("up", (f["ff"], W)), ("down", (W, f["ff"]))):
                mat(p + "mlp." + n, *shape); vec(p + "mlp." + n + ".b", shape[0])
        if ns:
            mat(p + "side.gate", ns, W, gain=1.5); mat(p + "side.proj", W, ns); vec(p + "side.norm", W, mid=0.7)
    return out


def bf16_round(a):
    """float32 -> the nearest bfloat16 (ties to even), back as float32"""
    b = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    b = ((b + 0x7FFF + ((b >> 16) & 1)) >> 16) << 16
    return b.astype(np.uint32).view(np.float32).reshape(np.shape(a))


def write_checkpoint(path, cfg, W):
    """config.json + model.safetensors with the weights as bfloat16 (the caller's oracle should use bf16_round of W)"""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({k: v for k, v in cfg.items() if not k.startswith("_")}, f)
    header, blobs, at = {}, [], 0
    for name, a in W.items():
        raw = (np.ascontiguousarray(bf16_round(a), np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw); at += len(raw)
    hj = json.dumps(header).encode()
    hj += b" " * (-len(hj) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(hj))); f.write(hj)
        for b in blobs:
            f.write(b)
