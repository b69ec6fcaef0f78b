"""Plain, slow statement of the latent-attention decoder (the "Dudilix" design), one function per mechanism, in float64
on the CPU.  The GPU tests compare the library with it; it shares no code with the library.

A sequence is evaluated whole: no cache, no chunks, no kernels.  Weights are a dict of float64 numpy arrays under the
checkpoint's tensor names; cfg is the parsed config.json.
"""
import math

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the pair table per token: a hash of (previous, current); the extra last row for a first token."""
    rows = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return rows


def embed(cfg, w, tokens):
    x = w["embed"][np.asarray(tokens)]
    bi = cfg.get("embedding", {}).get("bigram")
    if bi:
        x = x + w["bigram"][bigram_rows(tokens, bi["buckets"], bi["mul_prev"], bi["mul_cur"])]
    return x


def rotate_pairs(x, positions, base, dims):
    """Rotary positions, neighbouring dimensions (2i, 2i+1) as a pair, on the first `dims` of the last axis.
    x [..., tokens, d]."""
    out = x.copy()
    for i in range(dims // 2):
        a = np.asarray(positions, np.float64) * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a), np.sin(a)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def softmax_rows(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def causal_attention(q, k, v, scale):
    """q [H,T,dk], k [H,T,dk], v [H,T,dv] -> [H,T,dv]"""
    T = q.shape[1]
    s = np.matmul(q, np.swapaxes(k, 1, 2)) * scale
    s = np.where(np.tril(np.ones((T, T), bool)), s, -np.inf)
    return np.matmul(softmax_rows(s), v)


def latent_parts(h, w, p, mix, eps):
    """(normed latent c [T,r], rotated shared key part [T,rot])"""
    r = mix["kv_rank"]
    d = h @ w[p + "dkv"].T
    c = rms_norm(d[:, :r], w[p + "dkv.norm"], eps)
    kr = rotate_pairs(d[:, r:], np.arange(len(h)), mix["rot"]["base"], mix["rot"]["dims"])
    return c, kr


def latent_attention(h, w, p, mix, eps):
    """h [T,width] (already normed) -> [T,width]"""
    T, H, dim, rot, dv = len(h), mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dim + rot).transpose(1, 0, 2)
    q = np.concatenate([q[..., :dim], rotate_pairs(q[..., dim:], np.arange(T), mix["rot"]["base"], mix["rot"]["dims"])], -1)
    c, kr = latent_parts(h, w, p, mix, eps)
    k = (c @ w[p + "uk"].T).reshape(T, H, dim).transpose(1, 0, 2)
    k = np.concatenate([k, np.broadcast_to(kr, (H, T, rot))], -1)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv).transpose(1, 0, 2)
    o = causal_attention(q, k, v, mix["scale"]).transpose(1, 0, 2)
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[p + "o"].T


def gated_mlp(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def layer(x, w, i, spec, eps):
    n = "l%d." % i
    x = x + rms_norm(latent_attention(rms_norm(x, w[n + "norm1"], eps), w, n + "mix.", spec["mixer"], eps), w[n + "norm1b"], eps)
    if spec.get("mlp"):
        x = x + rms_norm(gated_mlp(rms_norm(x, w[n + "norm2"], eps), w, n + "mlp."), w[n + "norm2b"], eps)
    return x


def layer_order(cfg):
    """[(layer, starts a pass)] in the order they run."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        order += [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return order + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg, w, tokens, streams=None):
    """logits [T,vocab]; `streams` (a list) receives the residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x0 = x = embed(cfg, w, tokens)
    for i, starts in layer_order(cfg):
        if starts:
            x = np.concatenate([x, x0], -1) @ w["loop.in"].T
        x = layer(x, w, i, cfg["layers"][i], eps)
        if streams is not None:
            streams.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
