"""Plain, slow statement of the "Kulanex" decoder in float64 on the CPU, one function per mechanism: a gated delta rule with a
decay per key channel, a windowed attention beside a matrix memory, sparse feed-forwards, norms behind the sublayers.  The GPU
tests compare the library with it; it shares no code with the library.

A sequence is evaluated whole: no cache, no portions, no kernels; the recurrences are loops over tokens.  Weights are a dict of
float64 numpy arrays under the checkpoint's tensor names; cfg is the parsed config.json.
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_around_zero(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def short_conv(u, w):
    """u [T, C], w [C, taps]: causal, per channel; the last column of w meets the current token."""
    T, taps = len(u), w.shape[1]
    y = np.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def rotary_frequencies(rot):
    """One angle per position for every rotated pair; long wavelengths are stretched when rot has a scaling."""
    out = []
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif not wave < sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_pairs(x, rot):
    """x [T, heads, dim]: neighbouring dimensions (2i, 2i+1) turn together by position * frequency i."""
    out = x.copy()
    p = np.arange(len(x), dtype=np.float64)[:, None]
    for i, f in enumerate(rotary_frequencies(rot)):
        c, s = np.cos(p * f), np.sin(p * f)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def window_mask(T, size, keep_first):
    """[query, key]: the last `size` tokens (the query's own among them) and the sequence's first keep_first."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def masked_softmax(s, mask):
    s = np.where(mask, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def attention_parts(h, w, p, m, eps):
    """queries [T, H, dim], keys and values [T, G, dim] of the windowed attention"""
    T = len(h)
    q = short_conv(h @ w[p + "q"].T, w[p + "q.conv"])
    k = short_conv(h @ w[p + "k"].T, w[p + "k.conv"])
    v = k.reshape(T, m["kv_heads"], m["dim"])
    q = (rms(q, eps) * w[p + "q.norm"]).reshape(T, m["heads"], m["dim"])
    k = (rms(k, eps) * w[p + "k.norm"]).reshape(T, m["kv_heads"], m["dim"])
    return rotate_pairs(q, m["rot"]), rotate_pairs(k, m["rot"]), v


def window_attention(h, w, p, m, eps):
    T, H, G = len(h), m["heads"], m["kv_heads"]
    q, k, v = attention_parts(h, w, p, m, eps)
    mask = window_mask(T, m["mask"]["size"], m["mask"]["keep_first"])
    out = np.zeros((T, H, m["vdim"]))
    for i in range(H):
        g = i // (H // G)
        out[:, i] = masked_softmax(q[:, i] @ k[:, g].T * m["scale"], mask) @ v[:, g]
    return out.reshape(T, -1) @ w[p + "o"].T


def matrix_memory_cell(q, k, v, i, f):
    """q, k [T, H, d], v [T, H, dv], log input and log forget gates [T, H] -> [T, H, dv]"""
    T, H, d = k.shape
    S, n, m = np.zeros((H, d, v.shape[2])), np.zeros((H, d)), np.zeros(H)
    out = np.zeros(v.shape)
    for t in range(T):
        new = np.maximum(f[t] + m, i[t])
        keep, put = np.exp(f[t] + m - new), np.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + put[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + put[:, None] * k[t]
        den = np.maximum(np.abs((n * q[t]).sum(-1)), np.exp(-m)) + 1e-6
        out[t] = np.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def matrix_memory_gates(h, w, p, cap):
    i = cap * np.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = -softplus(-cap * np.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def matrix_memory(h, w, p, m, eps):
    T, H = len(h), m["heads"]
    q = (h @ w[p + "q"].T).reshape(T, H, m["dim"]) * m["dim"] ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, m["dim"])
    v = (h @ w[p + "v"].T).reshape(T, H, m["vdim"])
    i, f = matrix_memory_gates(h, w, p, m["gate_cap"])
    o = rms(matrix_memory_cell(q, k, v, i, f), eps).reshape(T, -1)
    return (o * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    return m["left_scale"] * window_attention(h, w, p + "left.", m["left"], eps) + m["right_scale"] * matrix_memory(h, w, p + "right.", m["right"], eps)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_cell(q, k, v, g, beta):
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H] -> [T, H, dv]"""
    T, H, d = k.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def delta_decays(h, w, p, m):
    a = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    return np.exp(-np.exp(w[p + "A_log"])[:, None] * softplus(a).reshape(len(h), m["heads"], m["dim"]))


def channel_delta(h, w, p, m, eps):
    T, H, G = len(h), m["heads"], m["kv_heads"]
    q = silu(short_conv(h @ w[p + "q"].T, w[p + "q.conv"])).reshape(T, G, m["dim"])
    k = silu(short_conv(h @ w[p + "k"].T, w[p + "k.conv"])).reshape(T, G, m["dim"])
    v = silu(short_conv(h @ w[p + "v"].T, w[p + "v.conv"])).reshape(T, H, m["vdim"])
    q = np.repeat(unit(q) * m["dim"] ** -0.5, H // G, axis=1)
    k = np.repeat(unit(k), H // G, axis=1)
    o = delta_cell(q, k, v, delta_decays(h, w, p, m), sigmoid(h @ w[p + "b"].T))
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, m["vdim"])
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, -1) @ w[p + "o"].T


def chosen_experts(h, w, p, router):
    """(experts [T, top], their scores)"""
    s = sigmoid(h @ w[p + "router"].T)
    top = np.argsort(-s, axis=1, kind="stable")[:, :router["top"]]
    return top, np.take_along_axis(s, top, 1)


def experts(h, w, p, mlp):
    top, score = chosen_experts(h, w, p, mlp["router"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, s in zip(top[t], score[t]):
            x = s * h[t]
            n = p + "e%d." % e
            out[t] += w[n + "down"] @ (silu(w[n + "gate"] @ x) * (w[n + "up"] @ x))
    return out


MIXERS = {"parallel": parallel, "channel_delta": channel_delta}


def layer(x, w, i, spec, eps, mult):
    n = "l%d." % i
    x = x + mult * norm_around_zero(MIXERS[spec["type"]](x, w, n + "mix.", spec["mixer"], eps), w[n + "norm1"], eps)
    if spec.get("mlp"):
        x = x + mult * norm_around_zero(experts(x, w, n + "mlp.", spec["mlp"]), w[n + "norm2"], eps)
    return x


def forward(cfg, w, tokens, streams=None):
    """logits [T, vocab]; `streams` (a list) receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    for i, spec in enumerate(cfg["layers"]):
        x = layer(x, w, i, spec, eps, cfg["residual_mult"])
        if streams is not None:
            streams.append(x)
    return norm_around_zero(x, w["final.norm"], eps) @ w["head"].T
