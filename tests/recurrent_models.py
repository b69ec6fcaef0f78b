"""Small random models of the "Kulanex" design: configurations and weights for the tests."""
import numpy as np

from latent_models import to_bf16

SCALING = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 256}


def delta(heads, kv_heads, dim, vdim, conv=4, ranks=(8, 8)):
    """`ranks`: of the low-rank maps of decays and gates; the config leaves them to the tensors."""
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "_ranks": ranks}


def window(heads, kv_heads, dim, size, keep_first=0, conv=4, rot_dims=None, base=10000.0, scale=None, scaling=SCALING):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": conv, "scale": dim ** -0.5 if scale is None else scale,
            "mask": {"size": size, "keep_first": keep_first}, "rot": {"base": base, "dims": rot_dims or dim // 2 * 2, "scaling": scaling}}


def memory(heads, dim, vdim, gate_cap=10.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def parallel(left, right, left_scale=0.7, right_scale=1.3):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(width, vocab, layers, eps=1e-5, residual_mult=0.4):
    """layers: [(mixer layer, feed-forward or None)]"""
    return {"architecture": "Kulanex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": residual_mult,
            "layers": [dict(m, mlp=f) for m, f in layers]}


def public(cfg):
    """what config.json holds"""
    return dict(cfg, layers=[{k: v for k, v in l.items() if not k.startswith("_")} for l in cfg["layers"]])


def shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        out[p + "norm1"] = (W,)
        if l["type"] == "channel_delta":
            H, k, v = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            ra, rg = l["_ranks"]
            x = p + "mix."
            out.update({x + "q": (k, W), x + "q.conv": (k, m["conv"]), x + "k": (k, W), x + "k.conv": (k, m["conv"]), x + "v": (v, W),
                        x + "v.conv": (v, m["conv"]), x + "b": (H, W), x + "A_log": (H,), x + "norm": (m["vdim"],), x + "a1": (ra, W),
                        x + "a2": (H * m["dim"], ra), x + "dt_bias": (H * m["dim"],), x + "g1": (rg, W), x + "g2": (v, rg), x + "o": (W, v)})
        else:
            a, r = m["left"], m["right"]
            q, k = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
            x = p + "mix.left."
            out.update({x + "q": (q, W), x + "k": (k, W), x + "q.norm": (q,), x + "k.norm": (k,), x + "q.conv": (q, a["conv"]),
                        x + "k.conv": (k, a["conv"]), x + "o": (W, q)})
            d, v = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            x = p + "mix.right."
            out.update({x + "q": (d, W), x + "k": (d, W), x + "v": (v, W), x + "g": (v, W), x + "o": (W, v), x + "norm": (v,),
                        x + "i": (r["heads"], W), x + "i.b": (r["heads"],), x + "f": (r["heads"], W), x + "f.b": (r["heads"],)})
        if l["mlp"]:
            f, E = l["mlp"]["expert"]["ff"], l["mlp"]["router"]["experts"]
            out[p + "norm2"] = (W,)
            for e in range(E):
                x = p + "mlp.e%d." % e
                out.update({x + "gate": (f, W), x + "up": (f, W), x + "down": (W, f)})
            out[p + "mlp.router"] = (E, W)
    return out


def weights(cfg, seed, steady=True):
    """Random weights that are bf16 values, as float64: name -> array.

    steady: the routers read a few dimensions of the stream that no sublayer writes (their norm weights there are -1), so a
    token's experts do not depend on rounding."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    quiet = max(4, W // 8)
    out = {}
    for name, sh in sorted(shapes(cfg).items()):
        last = name.split(".")[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            a = 0.3 * rng.standard_normal(sh)
            if steady and name != "final.norm":
                a[:quiet] = -1.0
        elif last == "norm":
            a = 1.0 + 0.3 * rng.standard_normal(sh)
        elif last == "conv":
            a = rng.standard_normal(sh) * sh[1] ** -0.5
        elif last == "A_log":
            a = rng.uniform(-4.0, 0.0, sh)
        elif last == "dt_bias":
            a = rng.uniform(-4.0, -1.0, sh)
        elif last == "b" and len(sh) == 1:
            a = rng.uniform(2.0, 6.0, sh) if name.endswith("f.b") else rng.uniform(-1.0, 0.5, sh)
        elif name == "embed":
            a = rng.standard_normal(sh)
        elif last == "router":
            a = rng.standard_normal(sh) * sh[1] ** -0.5
            if steady:
                a[:, quiet:] = 0.0
                a *= 2.0
        else:
            a = rng.standard_normal(sh) * sh[1] ** -0.5
        out[name] = to_bf16(a)[1]
    return out
