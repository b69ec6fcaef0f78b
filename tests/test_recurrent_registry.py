"""Model registry and the plain statement of the recurrent design: host code, no GPU."""
import importlib
import json
import math

import numpy as np
import pytest

import latent_models as L
import plain_recurrent as P
import recurrent_models as R

mynn = importlib.import_module("my-nn-engine_amd")

CFG = R.config(88, 200, [
    (R.delta(6, 3, 20, 28, conv=3, ranks=(5, 70)), R.moe(40, 5, 2)),
    (R.parallel(R.window(4, 2, 24, 9, 2, conv=2, rot_dims=10), R.memory(3, 18, 30)), None),
    (R.parallel(R.window(2, 1, 40, 30, conv=5), R.memory(1, 8, 12)), R.moe(64, 3, 1))])


def write(tmp_path, cfg, w=None, name="m"):
    d = tmp_path / name
    if w is not None:
        return L.write_checkpoint(d, R.public(cfg), w)
    d.mkdir()
    (d / "config.json").write_text(json.dumps(R.public(cfg)))
    return d


def test_config_and_checkpoint_give_tensors_and_states(tmp_path):
    a = mynn.Arch(write(tmp_path, CFG, R.weights(CFG, 1)))
    assert a.name == "Kulanex"
    assert dict(a.tensors()) == R.shapes(CFG)
    c = a.config(mynn.BF16, 128, seq_q=7, batch=2)
    assert (c.hidden, c.vocab, c.max_seq, c.seq_q, c.batch, c.arch) == (88, 200, 128, 7, 2, a.id)
    # rows: keys and values of the two attentions (heads padded to 32), the token history; then a block per sequence and layer
    assert a.state_row_bytes(mynn.BF16) == [2 * 2 * 32 * 2, 2 * 64 * 2, 4, 0, 0, 0]
    assert a.state_row_bytes(mynn.F32)[:3] == [2 * 2 * 32 * 4, 2 * 64 * 4, 4]
    d = 6 * 28 * 20 + 3 * (2 * 3 * 20 + 6 * 28)                    # memory, last inputs of the convolutions
    p1 = 3 * 31 * 20 + 4 + 2 * (4 + 2) * 32                        # memory and normaliser, maxima, last inputs
    p2 = 1 * 13 * 8 + 4 + 5 * (2 + 1) * 64
    assert a.state_seq_bytes() == [0, 0, 0, 4 * d, 4 * p1, 4 * p2]


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][1].update(type="something_else"), "mixer 'something_else'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "feed-forward 'dense'"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "key/value heads"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top 6 of 5"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(vdim=32), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "rotated dimensions"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("low"), "low"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c.pop("residual_mult"), "residual_mult"),
    (lambda c: c.update(layers=[]), "no layers"),
])
def test_bad_configs_are_named(tmp_path, change, text):
    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    with pytest.raises(mynn.MynnError, match=text):
        mynn.Arch(write(tmp_path, cfg, R.weights(CFG, 1)))


def test_ranks_need_the_checkpoint(tmp_path):
    with pytest.raises(mynn.MynnError, match="l0.mix.a1"):
        mynn.Arch(write(tmp_path, CFG))
    w = R.weights(CFG, 1)
    del w["l0.mix.g1"]
    with pytest.raises(mynn.MynnError, match="l0.mix.g1"):
        mynn.Arch(write(tmp_path, CFG, w, "n"))


# ---- the plain statement agrees with itself ---------------------------------------------------------------------------
def test_plain_prefix_property():
    w = R.weights(CFG, 5, steady=False)
    toks = np.random.default_rng(5).integers(0, CFG["vocab"], 40)
    full = P.forward(CFG, w, toks)
    assert np.allclose(P.forward(CFG, w, toks[:23]), full[:23], rtol=1e-10, atol=1e-10)


def test_plain_convolution_and_window():
    u = np.arange(1.0, 6.0)[:, None]
    assert P.short_conv(u, np.array([[10.0, 1.0]])).ravel().tolist() == [1, 12, 23, 34, 45]
    m = P.window_mask(6, 2, 1)
    assert [np.flatnonzero(r).tolist() for r in m] == [[0], [0, 1], [0, 1, 2], [0, 2, 3], [0, 3, 4], [0, 4, 5]]


def test_plain_frequencies_take_every_branch():
    rot = {"base": 100.0, "dims": 16, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}}
    plain = P.rotary_frequencies({"base": 100.0, "dims": 16})
    f = P.rotary_frequencies(rot)
    waves = [2 * math.pi / x for x in plain]
    kept, cut = [w < 16 for w in waves], [w > 64 for w in waves]
    assert any(kept) and any(cut) and not all(a or b for a, b in zip(kept, cut))
    for x, y, a, b in zip(plain, f, kept, cut):
        assert y == x if a else y == x / 8 if b else x / 8 < y < x


def test_plain_memory_is_its_unstabilised_sum():
    """with the maxima taken out, the read-out is the gated sum of k v^T over the larger of |n . q| and 1"""
    rng = np.random.default_rng(9)
    T, H, d, v = 12, 2, 5, 3
    q, k, val = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, v))
    i, f = rng.standard_normal((T, H)), -P.softplus(-rng.standard_normal((T, H)))
    got = P.matrix_memory_cell(q, k, val, i, f)
    for t in range(T):
        for h in range(H):
            a = [math.exp(i[s, h] + f[s + 1:t + 1, h].sum()) * (k[s, h] @ q[t, h]) for s in range(t + 1)]
            want = sum(x * val[s, h] for s, x in enumerate(a)) / max(abs(sum(a)), 1.0)
            assert np.allclose(got[t, h], want, rtol=1e-4, atol=1e-5)


def test_plain_delta_rule_replaces_what_a_key_held():
    e = np.eye(3)
    k = np.array([[e[0]], [e[1]], [e[0]]])
    v = np.array([[[1.0, 2.0]], [[3.0, 4.0]], [[5.0, 6.0]]])
    one = np.ones((3, 1))
    out = P.delta_cell(np.array([[e[0]], [e[0]], [e[0] + e[1]]]), k, v, np.ones((3, 1, 3)), one)
    assert np.allclose(out[:, 0], [[1, 2], [1, 2], [5 + 3, 6 + 4]])
    out = P.delta_cell(k, k, v, np.array([[[1, 1, 1]], [[0.5, 1, 1]], [[0.5, 1, 1]]], float), one * 0.5)  # beta 0.5, a channel that decays
    assert np.allclose(out[2, 0], 0.25 * 0.5 * v[0, 0] + 0.5 * (v[2, 0] - 0.25 * 0.5 * v[0, 0]))


def test_plain_experts_weigh_their_input():
    cfg = R.moe(6, 4, 2)
    rng = np.random.default_rng(2)
    w = {"router": rng.standard_normal((4, 5))}
    for e in range(4):
        w.update({"e%d.gate" % e: rng.standard_normal((6, 5)), "e%d.up" % e: rng.standard_normal((6, 5)), "e%d.down" % e: rng.standard_normal((5, 6))})
    h = rng.standard_normal((1, 5))
    s = 1 / (1 + np.exp(-(w["router"] @ h[0])))
    want = 0
    for e in sorted(range(4), key=lambda e: -s[e])[:2]:
        x = s[e] * h[0]
        g = w["e%d.gate" % e] @ x
        want = want + w["e%d.down" % e] @ (g / (1 + np.exp(-g)) * (w["e%d.up" % e] @ x))
    assert np.allclose(P.experts(h, w, "", cfg)[0], want)
