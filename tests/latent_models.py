"""Small random models of the latent-attention design: configurations, weights and checkpoint directories for the tests."""
import json
import os
import struct

import numpy as np


def mixer(heads, dim, rot_dim, vdim, kv_rank, scale=None, base=10000.0, rot_dims=None):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
            "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dims or rot_dim}}


def config(width, vocab, layers, loop=None, bigram=None, eps=1e-5, logit_scale=1.0):
    """layers: [(mixer, ff or None)]"""
    cfg = {"architecture": "Dudilix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "embedding": {},
           "layers": [{"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers]}
    if bigram:
        cfg["embedding"]["bigram"] = {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    if cfg["embedding"].get("bigram"):
        out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    if cfg.get("loop"):
        out["loop.in"] = (W, 2 * W)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H = m["heads"]
        out.update({p + "norm1": (W,), p + "norm1b": (W,), p + "mix.q": (H * (m["dim"] + m["rot_dim"]), W),
                    p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], W), p + "mix.dkv.norm": (m["kv_rank"],),
                    p + "mix.uk": (H * m["dim"], m["kv_rank"]), p + "mix.uv": (H * m["vdim"], m["kv_rank"]), p + "mix.g": (H, W),
                    p + "mix.o": (W, H * m["vdim"])})
        if l["mlp"]:
            F = l["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.gate": (F, W), p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    return out


def to_bf16(a):
    """f64 -> (bit patterns, the values they stand for), round to nearest even"""
    u = np.asarray(a, np.float32).view(np.uint32).astype(np.uint64)
    bits = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)
    return bits, (bits.astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def weights(cfg, seed):
    """Random weights that are bf16 values, as float64: name -> array"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, sh in sorted(shapes(cfg).items()):
        if len(sh) == 1:
            a = 1.0 + 0.3 * rng.standard_normal(sh)
        elif name in ("embed", "bigram"):
            a = rng.standard_normal(sh)
        else:
            a = rng.standard_normal(sh) * sh[1] ** -0.5
        out[name] = to_bf16(a)[1]
    return out


def write_checkpoint(directory, cfg, w):
    """config.json + model.safetensors (bf16)"""
    os.makedirs(str(directory), exist_ok=True)
    header, blobs, off = {}, [], 0
    for name, a in w.items():
        raw = to_bf16(a)[0].tobytes()
        header[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [off, off + len(raw)]}
        off += len(raw)
        blobs.append(raw)
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(str(directory), "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    with open(os.path.join(str(directory), "config.json"), "w") as f:
        json.dump(cfg, f)
    return str(directory)


def row_errors(got, want):
    """per row: RMS over the vocabulary of the difference, means taken off, relative to the RMS of the wanted row"""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    c = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1) / (c ** 2).mean(-1))
