"""Float64 numpy restatement of the Ripupel design, one function per mechanism, whole sequence at once with explicit loops over time.

No cache, no state object, no code shared with the package: the recurrence is written as a recurrence, the convolution as a sum over earlier positions,
attention with full keys and values of every head and a full score matrix, every expert run on the tokens that chose it.  `forward(cfg, w, tokens)`
returns the logits of every position and the residual stream after every layer.  `w` maps checkpoint tensor names to float arrays; `cfg` is the
dictionary of config.json.
"""
import json
import math
import os
import struct

import numpy as np


def layer_norm(x, w, eps):
    """weight, no bias"""
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w


def rms_unit(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.where(z > 30.0, z, np.log1p(np.exp(np.minimum(z, 30.0))))


def embed(cfg, w, tokens):
    return w["embed"][np.asarray(tokens)] * float((cfg.get("embedding") or {}).get("scale", 1.0))


# ------------------------------------------------------------------------------------------------ the gated linear recurrence
def causal_conv(u, taps_w, bias):
    """[T, C] through [C, taps]; the last column is the current token's, zeros before the start"""
    T, taps = len(u), taps_w.shape[1]
    out = np.tile(bias, (T, 1)).astype(np.float64)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += taps_w[:, j] * u[s]
    return out


def block_gate(u, mats, bias):
    """sigmoid of a block-diagonal projection: part b of u through mats[b] [out, in]"""
    B = len(mats)
    parts = np.split(u, B, axis=-1)
    return sigmoid(np.concatenate([p @ m.T + b for p, m, b in zip(parts, mats, bias)], axis=-1))


def decay_log(r, lam):
    return -8.0 * r * softplus(lam)


def input_factor(log_a):
    return np.sqrt(1.0 - np.exp(2.0 * log_a))


def gated_recurrence(u, r, i, lam):
    la = decay_log(r, lam)
    a, b = np.exp(la), input_factor(la) * i * u
    S, out = np.zeros(u.shape[1]), np.zeros_like(u)
    for t in range(len(u)):
        S = a[t] * S + b[t]
        out[t] = S
    return out


def mixer_rglru(m, w, p, h):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r = block_gate(u, w[p + "ra"], w[p + "ra.b"])
    i = block_gate(u, w[p + "ri"], w[p + "ri.b"])
    return (gated_recurrence(u, r, i, w[p + "lam"]) * y) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ attention through a latent
def rotate(x, base):
    """[T, ..., d]: pairs (i, i + d / 2), angle position * base^(-2 i / d)"""
    T, d = x.shape[0], x.shape[-1]
    half = d // 2
    ang = np.arange(T)[:, None] * np.array([base ** (-2.0 * i / d) for i in range(half)])
    shape = (T,) + (1,) * (x.ndim - 2) + (half,)
    c, s = np.cos(ang).reshape(shape), np.sin(ang).reshape(shape)
    a, b = x[..., :half], x[..., half:]
    return np.concatenate([a * c - b * s, b * c + a * s], axis=-1)


def latent_rows(m, w, p, h, eps):
    """the latent of every token and the rotated key part shared by the heads"""
    R = m["kv_rank"]
    z = h @ w[p + "dkv"].T
    return rms_unit(z[:, :R], eps) * w[p + "dkv.norm"], rotate(z[:, R:], m["rot"]["base"])


def sink_softmax(s, sink):
    """rows of scores (masked ones are -inf); the sink is one more term of the denominator"""
    mx = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - mx)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - mx))


def latent_attention(q, kn, kr, v, scale, sink):
    """q [T, H, dim + rot], kn [T, H, dim], kr [T, rot], v [T, H, vdim] -> [T, H, vdim]"""
    T, H, dim = kn.shape
    mask = np.where(np.tril(np.ones((T, T), bool)), 0.0, -np.inf)
    out = np.zeros((T, H, v.shape[-1]))
    for h in range(H):
        s = (q[:, h, :dim] @ kn[:, h].T + q[:, h, dim:] @ kr.T) * scale + mask
        out[:, h] = sink_softmax(s, sink[h]) @ v[:, h]
    return out


def output_gate(o, h, wg):
    return o * sigmoid(h @ wg.T)


def mixer_latent(m, w, p, h, c, kr):
    T, H, dim, rot = len(h), m["heads"], m["dim"], m["rot_dim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dim + rot)
    q = np.concatenate([q[..., :dim], rotate(q[..., dim:], m["rot"]["base"])], axis=-1)
    kn = (c @ w[p + "uk"].T).reshape(T, H, dim)
    v = (c @ w[p + "uv"].T).reshape(T, H, m["vdim"])
    o = latent_attention(q, kn, kr, v, m["scale"], w[p + "sink"]).reshape(T, -1)
    return output_gate(o, h, w[p + "g"]) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def gated_ff(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, wr, top):
    """ids and weights of every token's experts: sigmoid scores, the largest first, not renormalised"""
    s = sigmoid(h @ wr.T)
    ids = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=-1)


def experts_ff(h, w, p, top):
    ids, wt = route(h, w[p + "router"], top)
    out = np.zeros_like(h)
    for k in range(top):
        for e in np.unique(ids[:, k]):
            sel = ids[:, k] == e
            out[sel] += gated_ff(h[sel] * wt[sel, k:k + 1], w, p + f"e{e}.")      # the weight multiplies the expert's INPUT
    return out


def forward(cfg, W, tokens):
    w = {k: np.asarray(v, np.float64) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = embed(cfg, w, tokens)
    streams, kept = [], {}
    for i, lc in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lc["mixer"], lc.get("mlp")
        h = layer_norm(x, w[p + "norm1"], eps)
        if lc["type"] == "rglru":
            y = mixer_rglru(m, w, p + "mix.", h)
        else:
            src = m.get("kv_from")
            if src is None:
                kept[i] = latent_rows(m, w, p + "mix.", h, eps)
            y = mixer_latent(m, w, p + "mix.", h, *kept[i if src is None else src])
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        if f is not None:
            h = layer_norm(x, w[p + "norm2"], eps)
            y = gated_ff(h, w, p + "mlp.") if f["kind"] == "dense" else experts_ff(h, w, p + "mlp.", f["router"]["top"])
            x = x + layer_norm(y, w[p + "norm2b"], eps)
        streams.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T, np.stack(streams)


# ------------------------------------------------------------------------------------------------ configurations and weights of the tests
def latent(heads, dim, rot_dim, vdim, kv_rank, scale=None, base=1e4, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale,
         "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def rglru(width, blocks, conv):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def make_config(width, vocab, layers, eps=1e-5, embed_scale=1.0):
    return {"architecture": "Ripupel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": layers}


def random_weights(cfg, seed):
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}

    def mat(name, *shape, gain=1.0):
        out[name] = (rng.standard_normal(shape) * gain / math.sqrt(shape[-1])).astype(np.float32)

    def vec(name, *shape, mid=0.0, amp=0.2):
        out[name] = (mid + amp * rng.standard_normal(shape)).astype(np.float32)
    out["embed"] = (rng.standard_normal((V, W)) * 0.8).astype(np.float32)
    vec("final.norm", W, mid=1.0)
    for i, lc in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lc["mixer"], lc.get("mlp")
        vec(p + "norm1", W, mid=1.0); vec(p + "norm1b", W, mid=0.7)
        q = p + "mix."
        if lc["type"] == "rglru":
            D, B = m["width"], m["blocks"]
            mat(q + "y", D, W); vec(q + "y.b", D); mat(q + "x", D, W); vec(q + "x.b", D)
            out[q + "conv"] = (rng.standard_normal((D, m["conv"])) * 0.6).astype(np.float32)
            vec(q + "conv.b", D)
            for n in ("ra", "ri"):
                mat(q + n, B, D // B, D // B, gain=1.5); vec(q + n + ".b", B, D // B, amp=0.7)
            vec(q + "lam", D, mid=-3.5, amp=2.0)
            mat(q + "o", W, D)
        else:
            H, d, rd, dv, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            mat(q + "q", H * (d + rd), W, gain=2.0)
            if m.get("kv_from") is None:
                mat(q + "dkv", R + rd, W); vec(q + "dkv.norm", R, mid=1.0)
            mat(q + "uk", H * d, R); mat(q + "uv", H * dv, R); vec(q + "sink", H, amp=1.5)
            mat(q + "g", H * dv, W); mat(q + "o", W, H * dv)
        if f is not None:
            vec(p + "norm2", W, mid=1.0); vec(p + "norm2b", W, mid=0.7)
            if f["kind"] == "dense":
                mat(p + "mlp.gate", f["ff"], W); mat(p + "mlp.up", f["ff"], W); mat(p + "mlp.down", W, f["ff"])
            else:
                mat(p + "mlp.router", f["router"]["experts"], W, gain=2.0)
                for e in range(f["router"]["experts"]):
                    F = f["expert"]["ff"]
                    mat(p + f"mlp.e{e}.gate", F, W, gain=1.5); mat(p + f"mlp.e{e}.up", F, W, gain=1.5); mat(p + f"mlp.e{e}.down", W, F)
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
        json.dump(cfg, f)
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
