"""The latent-attention design ("Dudilix") on the GPU against its plain statement (plain_latent.py): f32 executors closely,
bf16 executors within bf16 rounding.  Small random models of many shapes, through the same entry points as the Llama graph."""
import importlib
import json
import os
import subprocess

import numpy as np
import pytest

import latent_models as L
import plain_latent as P
from conftest import GOLDEN, ROOT

pytestmark = pytest.mark.gpu
mynn = importlib.import_module("my-nn-engine_amd")

F32, BF16 = mynn.F32, mynn.BF16
TOL = {F32: 2e-5, BF16: 4e-2}
DTYPES = [pytest.param(F32, id="f32"), pytest.param(BF16, id="bf16")]

# shapes: nothing divides anything; several mixers in one model; loops at the front, the end, over everything
MODELS = {
    "odd": L.config(100, 333, [(L.mixer(3, 24, 8, 16, 40), 70), (L.mixer(2, 32, 4, 48, 100), None), (L.mixer(1, 16, 16, 32, 8), 36)],
                    loop=(1, 3, 3), bigram=(77, 31, 5), eps=1e-3, logit_scale=3.5),
    "plain": L.config(128, 256, [(L.mixer(2, 64, 32, 64, 128, base=250000.0), 192)] * 2),
    "all_looped": L.config(72, 150, [(L.mixer(5, 40, 24, 24, 72), 96), (L.mixer(5, 40, 24, 24, 72), 50)], loop=(0, 2, 2), bigram=(11, 7, 3)),
    "wide_latent": L.config(160, 200, [(L.mixer(4, 128, 64, 128, 320, scale=0.02), 130)], bigram=(1, 1, 1)),
    "many_heads": L.config(192, 500, [(L.mixer(20, 16, 6, 80, 136, rot_dims=4), None), (L.mixer(20, 16, 6, 80, 136), 64)], loop=(1, 2, 2)),
    "one_pass_loop": L.config(64, 97, [(L.mixer(1, 8, 2, 8, 16), 24)] * 2, loop=(0, 1, 1), bigram=(1000, 113, 401), logit_scale=0.25),
}


class Case:
    """A model with its checkpoint and plain logits."""

    def __init__(self, path, cfg, seed):
        self.cfg, self.w, self.path = cfg, L.weights(cfg, seed), str(path)
        self.rng = np.random.default_rng(seed + 1000)

    def save(self):
        L.write_checkpoint(self.path, self.cfg, self.w)
        return self

    def tokens(self, n):
        return [int(t) for t in self.rng.integers(0, self.cfg["vocab"], n)]

    def want(self, toks):
        return P.forward(self.cfg, self.w, toks)


@pytest.fixture(scope="module", params=list(MODELS))
def case(request, tmp_path_factory):
    return Case(tmp_path_factory.mktemp(request.param), MODELS[request.param], len(request.param)).save()


def feed_all(session, toks, sizes):
    """every logit of toks, fed in portions of the given sizes (repeated)"""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        out.append(session.feed(toks[at:at + n], list(range(n))))
        at += n
        i += 1
    return np.concatenate(out)


def close(got, want, dt, factor=1.0):
    e = L.row_errors(got, want)
    assert np.isfinite(e).all() and e.max() <= factor * TOL[dt], (float(e.max()), int(e.argmax()))


# ---- whole models: every shape, prompts, portions, decoding --------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
def test_prompt_portions_and_token_by_token(case, dt):
    toks = case.tokens(150)
    want = case.want(toks)
    eng = mynn.Engine(case.path, dt, 512, prefill_rows=150)
    s = eng.session()
    for sizes in ([150], [1], [2], [3, 1, 31, 2], [33], [32, 64], [100, 2, 1]):
        close(feed_all(s, toks, sizes), want, dt)
        assert s.past_len == len(toks)
        s.reset()
    # only some logits, in gaps
    places = [0, 1, 40, 41, 99, 148]
    close(s.feed(toks, places), want[places], dt)
    s.close()
    eng.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_small_prompt_steps_cut_a_portion(case, dt):
    """a portion larger than the prompt executor's rows runs in several steps"""
    toks = case.tokens(90)
    eng = mynn.Engine(case.path, dt, 128, prefill_rows=37)
    s = eng.session()
    close(s.feed(toks, list(range(90))), case.want(toks), dt)
    s.close()
    eng.close()


# ---- mechanisms alone -------------------------------------------------------------------------------------------------------
def run_once(tmp_path, cfg, w, toks, dt, sizes):
    c = Case(tmp_path, cfg, 0)
    c.w = w
    c.save()
    eng = mynn.Engine(c.path, dt, 320)
    s = eng.session()
    got = feed_all(s, toks, sizes)
    s.close()
    eng.close()
    return got


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[40], [1], [7]])
def test_embedding_pairs_final_norm_and_scale(tmp_path, dt, sizes):
    """the mixer's output is zero, which the norm behind it leaves at zero: embedding and head remain"""
    cfg = L.config(80, 60, [(L.mixer(1, 8, 4, 8, 8), None)], bigram=(13, 1 << 30, 5), eps=0.05, logit_scale=-2.0)
    w = L.weights(cfg, 3)
    w["l0.mix.o"][:] = 0
    w["bigram"] *= 4  # a wrong pair row shows
    toks = [int(t) for t in np.random.default_rng(3).integers(0, 60, 40)]
    got = run_once(tmp_path, cfg, w, toks, dt, sizes)
    close(got, P.forward(cfg, w, toks), dt, 0.5)
    # (a first token has a row of its own: taking row 0 instead would show)
    wrong = dict(w, bigram=np.concatenate([w["bigram"][:-1], w["bigram"][:1]]))
    assert L.row_errors(P.forward(cfg, wrong, toks), P.forward(cfg, w, toks))[0] > 0.3


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[40], [1]])
def test_gated_feed_forward(tmp_path, dt, sizes):
    cfg = L.config(136, 90, [(L.mixer(1, 8, 4, 8, 8), 200)])
    w = L.weights(cfg, 4)
    w["l0.mix.o"][:] = 0
    w["l0.mlp.gate"] *= 4  # both ends of the activation
    toks = [int(t) for t in np.random.default_rng(4).integers(0, 90, 40)]
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), P.forward(cfg, w, toks), dt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[120], [1], [9]])
@pytest.mark.parametrize("what", ["rotation", "gates", "sharp"])
def test_latent_attention_alone(tmp_path, dt, sizes, what):
    cfg = L.config(96, 110, [(L.mixer(3, 32, 48, 40, 56, base=37.0), None)])
    w = L.weights(cfg, 6)
    mix = cfg["layers"][0]["mixer"]
    if what == "rotation":  # the scores are the rotated part's
        q = w["l0.mix.q"].reshape(3, 80, 96)
        q[:, :32] = 0
    if what == "gates":
        w["l0.mix.g"] *= 8
    if what == "sharp":     # close to one key per query, anywhere
        mix["scale"] = 2.5
    toks = [int(t) for t in np.random.default_rng(6).integers(0, 110, 120)]
    # (a sharp softmax magnifies the rounding of its scores)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), P.forward(cfg, w, toks), dt, 6.0 if what == "sharp" and dt == BF16 else 1.0)


@pytest.mark.parametrize("dt", DTYPES)
def test_loop_passes_have_caches_of_their_own(tmp_path, dt):
    cfg = L.config(64, 80, [(L.mixer(2, 16, 8, 16, 24), 40)] * 3, loop=(1, 2, 4), bigram=(9, 2, 3))
    w = L.weights(cfg, 8)
    w["loop.in"][:, 64:] *= 2  # the embedding's half counts
    toks = [int(t) for t in np.random.default_rng(8).integers(0, 80, 60)]
    want = P.forward(cfg, w, toks)
    for i, sizes in enumerate(([60], [1], [5])):
        close(run_once(tmp_path / str(i), cfg, w, toks, dt, sizes), want, dt)
    assert L.row_errors(P.forward(dict(cfg, loop={"start": 1, "stop": 2, "times": 3}), w, toks), want).max() > 0.1


# ---- kernel forms -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("heads,dim,rot,vdim,rank", [
    (2, 64, 24, 56, 64), (3, 100, 28, 64, 130), (1, 192, 64, 33, 64), (2, 32, 32, 128, 256), (4, 128, 64, 128, 512), (1, 160, 32, 100, 64),
    (17, 32, 32, 32, 200), (33, 16, 16, 16, 450), (2, 224, 64, 64, 64), (2, 32, 16, 160, 64), (1, 32, 128, 64, 64), (2, 32, 160, 64, 64), (2, 16, 8, 16, 600)])
def test_attention_forms(tmp_path, heads, dim, rot, vdim, rank):
    """bf16: every tile form of the prompt and the decode kernels, and the shapes beyond them"""
    cfg = L.config(128, 64, [(L.mixer(heads, dim, rot, vdim, rank), None)])
    w = L.weights(cfg, heads * 7 + dim)
    toks = [int(t) for t in np.random.default_rng(dim).integers(0, 64, 300)]
    want = P.forward(cfg, w, toks)
    for i, sizes in enumerate(([300], [270] + [1] * 30, [200, 20, 3, 2])):
        close(run_once(tmp_path / str(i), cfg, w, toks, BF16, sizes), want, BF16)


# ---- one key that matters, anywhere: page borders, tile borders, first tokens ---------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
def test_a_single_far_key_is_found(tmp_path, dt):
    """Query tokens whose attention sits on one earlier position; without that key the answer is another."""
    cfg = L.config(96, 400, [(L.mixer(4, 48, 8, 32, 64, scale=1.0), None)])
    c = Case(tmp_path, cfg, 21)
    for t in ("embed", "l0.mix.q"):
        c.w[t] = L.to_bf16(c.w[t] * 1.5)[1]
    c.save()
    base = c.tokens(330)
    eps, mix = cfg["norm"]["eps"], cfg["layers"][0]["mixer"]

    def weights_at(toks):  # softmax rows of the last token, [H, T]
        h = P.rms_norm(P.embed(cfg, c.w, toks), c.w["l0.norm1"], eps)
        lat, kr = P.latent_parts(h, c.w, "l0.mix.", mix, eps)
        T = len(toks)
        q = (h[-1] @ c.w["l0.mix.q"].T).reshape(4, 1, 56)
        q = np.concatenate([q[..., :48], P.rotate_pairs(q[..., 48:], [T - 1], mix["rot"]["base"], 8)], -1)
        k = (lat @ c.w["l0.mix.uk"].T).reshape(T, 4, 48).transpose(1, 0, 2)
        k = np.concatenate([k, np.broadcast_to(kr, (4, T, 8))], -1)
        return P.softmax_rows(np.matmul(q, k.transpose(0, 2, 1))[:, 0] * mix["scale"])

    eng = mynn.Engine(c.path, dt, 512, prefill_rows=300)
    s = eng.session()
    tried = 0
    for n in (65, 129, 193, 330):
        for p in (0, 1, 31, 32, 63, 64, 127, 128, 191, 192, 255, 256, n - 2):
            if p >= n - 1:
                continue
            # the query token, of the vocabulary, that looks at position p the hardest
            h = P.rms_norm(c.w["embed"], c.w["l0.norm1"], eps)
            q = (h @ c.w["l0.mix.q"].T).reshape(-1, 4, 56)[:, :, :48]
            lat, _ = P.latent_parts(h[base[:n - 1]], c.w, "l0.mix.", mix, eps)
            k = (lat @ c.w["l0.mix.uk"].T).reshape(n - 1, 4, 48)
            sc = np.einsum("vhd,khd->vhk", q, k)
            lead = sc[:, :, p] - np.delete(sc, p, axis=2).max(-1)
            toks = base[:n - 1] + [int(np.unravel_index(lead.argmax(), lead.shape)[0])]
            if weights_at(toks)[:, p].max() < 0.3:
                continue  # (no token singles this position out)
            tried += 1
            want = c.want(toks)[-1:]
            for sizes in ([n - 1, 1], [n], [n - 40, 40], [n - 2, 2]):
                if min(sizes) < 1:
                    continue
                at = 0
                for m in sizes:
                    got = s.feed(toks[at:at + m], [m - 1])
                    at += m
                s.reset()
                close(got, want, dt, 2.0)
            # without that key the answer is another
            if p % 64 == 0 and n < 200:
                assert L.row_errors(without_key(c, toks, p), want).max() > 0.1
    assert tried >= 20, tried
    s.close()
    eng.close()


def without_key(c, toks, p):
    """the plain logits of the last token when position p is left out of its (single-layer) attention"""
    orig = P.softmax_rows

    def masked(sc):
        sc = sc.copy()
        sc[:, -1, p] = -np.inf
        return orig(sc)

    P.softmax_rows = masked
    try:
        return c.want(toks)[-1:]
    finally:
        P.softmax_rows = orig


# ---- cache: pages, sessions, reuse, rewind ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
def test_sessions_share_pages_and_reuse_them(case, dt):
    """Two sessions grow in turns over one pool; one ends and its pages serve a third.  The logits do not depend on which
    pages a session holds (bit for bit), nor on what was there before."""
    a, b, c = case.tokens(140), case.tokens(75), case.tokens(200)
    eng = mynn.Engine(case.path, dt, 448, max_seq=256, prefill_rows=64)
    free0 = eng.free_rows
    one = eng.session()
    alone = {n: feed_all(one, t, [50, 3, 1, 1]) for n, t in (("a", a),)}
    one.reset()
    alone["b"] = feed_all(one, b, [30, 1])
    one.reset()
    alone["c"] = feed_all(one, c, [64, 1, 1, 2])
    one.reset()
    assert eng.free_rows == free0
    two = eng.session()
    got_a, got_b, ia, ib, i = [], [], 0, 0, 0
    while ia < len(a) or ib < len(b):
        n = [50, 3, 1, 1][i % 4]
        if ia < len(a):
            n = min(n, len(a) - ia)
            got_a.append(one.feed(a[ia:ia + n], list(range(n))))
            ia += n
        m = [30, 1][i % 2]
        if ib < len(b):
            m = min(m, len(b) - ib)
            got_b.append(two.feed(b[ib:ib + m], list(range(m))))
            ib += m
        i += 1
    assert np.array_equal(np.concatenate(got_a), alone["a"]) and np.array_equal(np.concatenate(got_b), alone["b"])
    close(alone["a"], case.want(a), dt)
    one.reset()                       # its pages go to the next session
    three = eng.session()
    got_c = feed_all(three, c, [64, 1, 1, 2])
    assert np.array_equal(got_c, alone["c"])
    close(got_c, case.want(c), dt)
    close(feed_all(two, b[:1], [1]), case.want(b + b[:1])[-1:], dt)  # the other one goes on unharmed
    for s in (one, two, three):
        s.close()
    assert eng.free_rows == free0
    eng.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_rewind_finds_the_previous_token(case, dt):
    toks, other = case.tokens(100), case.tokens(30)
    eng = mynn.Engine(case.path, dt, 128, page_rows=128)
    s = eng.session()
    s.feed(toks, [])
    s.past_len = 70
    close(s.feed(other, list(range(30))), case.want(toks[:70] + other)[70:], dt)
    s.past_len = 64
    close(s.feed(other[:1], [0]), case.want(toks[:64] + other[:1])[64:], dt)
    s.close()
    eng.close()


def test_a_full_pool_and_a_long_prompt_are_refused(tmp_path):
    c = Case(tmp_path, MODELS["plain"], 1).save()
    eng = mynn.Engine(c.path, BF16, 64, max_seq=1024, prefill_rows=256)  # 1 + 8 pages of 64 rows
    s = eng.session()
    with pytest.raises(mynn.MynnError, match="free in the pool"):
        s.feed(c.tokens(1000), [])
    s.reset()
    with pytest.raises(mynn.MynnError, match="exceed max_seq"):
        s.feed(c.tokens(1025), [])
    toks = c.tokens(80)
    close(s.feed(toks, list(range(80))), c.want(toks), BF16)
    s.close()
    eng.close()


# ---- executors by hand: batches in step, contiguous caches, profile -----------------------------------------------------------
def device_weights(c, dt):
    import torch

    t = {F32: torch.float32, BF16: torch.bfloat16}[dt]
    return {k: torch.tensor(v, dtype=t, device="cuda") for k, v in c.w.items()}


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("paged", [False, True])
def test_batch_in_step_equals_each_alone(case, dt, paged):
    arch = mynn.Arch(case.path)
    w = device_weights(case, dt)
    B, N, D = 3, 70, 6
    seqs = [case.tokens(N + D) for _ in range(B)]
    pool = pages = None
    if paged:
        pool = mynn.KvPool(B * 2 + 3, 64)
        pages = mynn.KvPages(pool, B, 128)
        state = mynn.layered_state(arch, dt, pool.n_pages * 64, fill=0xFF)  # NaN everywhere
    else:
        state = mynn.layered_state(arch, dt, B * 128, fill=0xFF)
    pre = mynn.LayeredDecoder(arch, w, dt, 128, seq_q=64, batch=B, state=state, kv_pages=pages)
    dec = mynn.LayeredDecoder(arch, w, dt, 128, batch=B, state=state, kv_pages=pages)
    got = [[] for _ in range(B)]
    for lo, hi in ((0, 40), (40, 60), (60, N)):
        _, lg = pre.step_rows([s[lo:hi] for s in seqs], hi - lo, lo, n_logits=hi - lo)
        for b in range(B):
            got[b].append(lg[b])
    for i in range(D):
        nxt, lg = dec.step_rows([s[N + i] for s in seqs], 1, N + i)
        assert nxt == [int(np.flatnonzero(lg[b, 0] == lg[b, 0].max())[-1]) for b in range(B)]
        for b in range(B):
            got[b].append(lg[b])
    for b in range(B):
        close(np.concatenate(got[b]), case.want(seqs[b]), dt)
    pre.close(), dec.close()
    if paged:
        pages.close(), pool.close()


def test_step_profile_names_its_launches(tmp_path):
    c = Case(tmp_path, MODELS["all_looped"], 2).save()
    arch = mynn.Arch(c.path)
    dec = mynn.LayeredDecoder(arch, device_weights(c, BF16), BF16, 128)
    # embedding + 4 layer runs of 7 launches + 2 pass starts + head + greedy token
    assert dec.stats() == dict(dec.stats(), launches_per_step=1 + 4 * 7 + 2 + 2, graph=True)
    names = [n for n, ms, _, _ in dec.profile_step(3, 0) if ms > 0]
    assert names.count("latent_attention") == 4 and names.count("gemv_loop_in") == 2 and names[-1] == "greedy_advance"
    dec.close()


# ---- generation -----------------------------------------------------------------------------------------------------------------
def plain_greedy(c, prompt, n):
    """(ids, smallest gap between the best and the second logit)"""
    toks, gap = list(prompt), np.inf
    for _ in range(n):
        l = c.want(toks)[-1]
        o = np.sort(l)
        gap = min(gap, (o[-1] - o[-2]) / np.std(l))
        toks.append(int(l.argmax()))
    return toks[len(prompt):], gap


@pytest.mark.parametrize("prefill_rows", [1, 16, 512])
def test_greedy_generation_follows_the_plain_model(case, prefill_rows):
    prompt = case.tokens(23)
    ids, gap = plain_greedy(case, prompt, 40)
    assert gap > 1e-4  # (f32 separates the two best tokens at every step)
    eng = mynn.Engine(case.path, F32, 128, prefill_rows=prefill_rows)
    s = eng.session()
    assert s.generate_ids(prompt, 40) == ids
    assert s.past_len == len(prompt) + 39
    # a second turn continues the same sequence; then from the start, with an end-of-sequence id
    assert s.generate_ids([ids[-1], 5], 3) == plain_greedy(case, prompt + ids + [5], 3)[0]
    s.close()
    stop = ids[9]
    s = eng.session(eos=stop)
    assert s.generate_ids(prompt, 40) == ids[:ids.index(stop) + 1]
    s.close()
    eng.close()


def test_long_decoding_in_graph_runs_matches_the_prompt_path(tmp_path):
    """300 tokens from the device-resident loop; the same tokens fed as a prompt must name every one of them"""
    c = Case(tmp_path, MODELS["odd"], 31).save()
    for dt in (F32, BF16):
        eng = mynn.Engine(c.path, dt, 512)
        s = eng.session()
        prompt = c.tokens(10)
        ids = s.generate_ids(prompt, 300)
        assert len(ids) == 300
        s.reset()
        lg = s.feed(prompt + ids[:-1], list(range(9, 309)))
        best = lg.max(-1)
        chosen = lg[np.arange(300), ids]
        assert ((best - chosen) / lg.std(-1) <= (1e-4 if dt == F32 else 0.1)).all()
        want = c.want(prompt + ids[:-1])[9:]
        close(lg, want, dt)
        s.close()
        eng.close()


# ---- the trace program ------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,dt", [("float32", F32), ("bfloat16", BF16)])
def test_trace_program(case, tmp_path, dtype, dt):
    a, b = case.tokens(90), case.tokens(40)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:60], "want": [59, 0, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[60:62], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[62:63], "want": [0]}], "end": ["nobody"]},
             {"step": 7, "entries": [{"id": "a", "tokens": a[63:], "want": [26]}, {"id": "b", "tokens": b[:1], "want": [0]}], "end": ["a"]},
             {"step": 8, "entries": [{"id": "b", "tokens": b[1:], "want": [38]}], "end": ["b"]},
             {"step": 9, "entries": [{"id": "a", "tokens": b[:3], "want": [0, 1, 2]}], "end": ["a"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", case.path, "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=90)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % s["step"] for s in steps]
    wa, wb = case.want(a), case.want(b)

    def rows(n):
        return np.fromfile(str(tmp_path / ("%d.f32" % n)), np.float32).reshape(-1, case.cfg["vocab"])

    close(rows(0), wa[[59, 0, 7]], dt)
    assert not (tmp_path / "1.f32").exists()
    close(rows(2), wa[[62]], dt)
    close(rows(7), np.stack([wa[89], wb[0]]), dt)
    close(rows(8), wb[[39]], dt)
    close(rows(9), wb[:3], dt)


# ---- the other models through the same engine --------------------------------------------------------------------------------
def test_llama_checkpoint_through_the_engine():
    gold = json.load(open(os.path.join(GOLDEN, "tiny-llama-random", "golden_ids.json")))
    for prefill_rows in (1, 8):
        eng = mynn.Engine(os.path.join(GOLDEN, "tiny-llama-random"), BF16, 64, prefill_rows=prefill_rows)
        s = eng.session()
        assert s.generate_ids(gold["prompt_ids"], 8) == gold["expected_new_ids"]
        s.reset()
        toks = gold["prompt_ids"] + gold["expected_new_ids"]
        lg = s.feed(toks[:-1], list(range(8)))
        assert lg.argmax(-1).tolist() == gold["expected_new_ids"]
        s.close()
        eng.close()
    with pytest.raises(mynn.MynnError):
        mynn.Engine(os.path.join(GOLDEN, "tiny-llama-random"), F32, 64)
