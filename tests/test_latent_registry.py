"""Model registry and the plain statement of the latent-attention design: host code, no GPU."""
import importlib
import json
import os

import numpy as np
import pytest

import latent_models as L
import plain_latent as P
from conftest import GOLDEN

mynn = importlib.import_module("my-nn-engine_amd")

CFG = L.config(100, 333, [(L.mixer(3, 24, 8, 16, 40), 70), (L.mixer(2, 32, 4, 48, 100), None), (L.mixer(1, 16, 16, 32, 8), 36)],
               loop=(1, 3, 3), bigram=(77, 31, 5))


def write(tmp_path, cfg, name="m"):
    d = tmp_path / name
    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    return d


def test_config_gives_the_tensors_and_caches(tmp_path):
    a = mynn.Arch(write(tmp_path, CFG))
    assert a.name == "Dudilix"
    assert dict(a.tensors()) == L.shapes(CFG)
    c = a.config(mynn.F32, 128, seq_q=7, batch=2)
    assert (c.hidden, c.vocab, c.max_seq, c.seq_q, c.batch, c.arch) == (100, 333, 128, 7, 2, a.id)
    # one cache per layer run (7 runs: layer 0, then layers 1 and 2 three times), then the token history
    rows = a.state_row_bytes(mynn.F32)
    one, two, three = (64 + 32) * 4, (128 + 32) * 4, (64 + 32) * 4  # latent to 64 values, rotated part to 32
    assert rows == [one] + [two, three] * 3 + [4]
    assert P.layer_order(CFG) == [(0, False), (1, True), (2, False), (1, True), (2, False), (1, True), (2, False)]


@pytest.mark.parametrize("change,text", [
    (lambda c: c.update(architecture="Unheard"), "no model of architecture"),
    (lambda c: c["layers"][1].update(type="something_else"), "mixer 'something_else'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "feed-forward 'sparse'"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][0]["mixer"].update(heads=2.5), "heads"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=12), "rotated dimensions"),
    (lambda c: c["loop"].update(start=3), "loop"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.update(layers=[], loop=None), "no layers"),
])
def test_bad_configs_are_named(tmp_path, change, text):
    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    with pytest.raises(mynn.MynnError, match=text):
        mynn.Arch(write(tmp_path, cfg))


def test_llama_configs_are_in_the_same_registry():
    a = mynn.Arch(os.path.join(GOLDEN, "tiny-llama-random"))
    c = a.config(mynn.BF16, 64)
    assert a.name == "LlamaForCausalLM" and c.arch == 0
    assert (c.n_layers, c.hidden, c.n_heads, c.n_kv_heads, c.head_dim, c.ffn, c.vocab) == (2, 16, 4, 4, 4, 64, 32000)
    assert a.state_row_bytes(mynn.BF16) == [4 * 4 * 2] * 4


def test_layered_models_refuse_what_they_do_not_have(tmp_path):
    a = mynn.Arch(write(tmp_path, CFG))
    for change in (dict(dtype=mynn.F16), dict(quant_kv_cache=1), dict(streaming_kv=1), dict(kv_page_rows=48), dict(seq_q=200)):
        c = a.config(mynn.BF16, 128)
        for k, v in change.items():
            setattr(c, k, v)
        assert mynn.lib().mynn_model_configure(c) != 0, change


# ---- the plain statement agrees with itself ---------------------------------------------------------------------------
def test_plain_prefix_property_and_absorbed_identity():
    w = L.weights(CFG, 5)
    rng = np.random.default_rng(5)
    toks = rng.integers(0, CFG["vocab"], 20)
    full = P.forward(CFG, w, toks)
    assert np.allclose(P.forward(CFG, w, toks[:13]), full[:13], rtol=1e-10, atol=1e-10)
    # (W_uk c) . q == c . (W_uk^T q): the scores of one head taken either way
    mix, p, eps = CFG["layers"][1]["mixer"], "l1.mix.", CFG["norm"]["eps"]
    h = rng.standard_normal((9, CFG["width"]))
    c, kr = P.latent_parts(h, w, p, mix, eps)
    q = (h @ w[p + "q"].T).reshape(9, mix["heads"], -1)[:, 1, :mix["dim"]]
    uk = w[p + "uk"][mix["dim"]:2 * mix["dim"]]
    assert np.allclose(q @ (c @ uk.T).T, (q @ uk) @ c.T, rtol=1e-10)


def test_plain_bigram_rows_and_rotation():
    assert P.bigram_rows([4, 9, 2], 7, 3, 5) == [7, (4 * 3 + 9 * 5) % 7, (9 * 3 + 2 * 5) % 7]
    x = np.array([[1.0, 0.0, 0.0, 2.0, 5.0]])
    y = P.rotate_pairs(x, [3], 100.0, 4)  # angles 3 and 3 * 100^-0.5
    assert np.allclose(y, [[np.cos(3), np.sin(3), -2 * np.sin(0.3), 2 * np.cos(0.3), 5.0]])
    assert np.allclose(P.gelu_tanh(np.array([0.0, 1.0, -1.0])), [0.0, 0.841192, -0.158808], atol=1e-6)
