"""The recurrent design ("Kulanex") on the GPU against its plain statement (plain_recurrent.py): f32 executors closely, bf16
executors within bf16 rounding.  Small random models of many shapes, through the same entry points as the other designs."""
import importlib
import json
import os
import subprocess

import numpy as np
import pytest

import latent_models as L
import plain_recurrent as P
import recurrent_models as R
from conftest import ROOT

pytestmark = pytest.mark.gpu
mynn = importlib.import_module("my-nn-engine_amd")

F32, BF16 = mynn.F32, mynn.BF16
# (largest row error, median row error).  A head's read-out is divided by its own root mean square, so a row where it nearly
# cancels magnifies the bf16 rounding of its parts: the median is the sharp bound there, and f32 throughout.
TOL = {F32: (3e-5, 1e-5), BF16: (0.15, 0.02)}
DTYPES = [pytest.param(F32, id="f32"), pytest.param(BF16, id="bf16")]

MODELS = {
    "mixed": R.config(88, 200, [
        (R.delta(6, 3, 20, 28, conv=3, ranks=(5, 70)), R.moe(40, 5, 2)),
        (R.parallel(R.window(4, 2, 24, 9, 2, conv=2, rot_dims=10), R.memory(3, 18, 30)), None),
        (R.parallel(R.window(2, 1, 40, 70, conv=5), R.memory(1, 8, 12)), R.moe(64, 3, 1))], eps=1e-4),
    "one_tap": R.config(64, 150, [
        (R.parallel(R.window(3, 3, 64, 33, 5, conv=1), R.memory(2, 64, 16, gate_cap=3.0), 1.0, 1.0), R.moe(24, 1, 1)),
        (R.delta(2, 2, 64, 64, conv=1, ranks=(64, 1)), R.moe(100, 7, 3))], residual_mult=1.0),
    "deltas": R.config(120, 99, [(R.delta(5, 1, 36, 52, conv=6, ranks=(16, 40)), None), (R.delta(4, 4, 8, 100), R.moe(33, 12, 4))], residual_mult=0.9),
    "wide_groups": R.config(136, 300, [
        (R.parallel(R.window(10, 2, 96, 50, 1, rot_dims=48, base=500.0), R.memory(2, 100, 40)), R.moe(72, 70, 8)),
        (R.parallel(R.window(6, 1, 128, 129, 64, scaling=None), R.memory(4, 4, 4)), R.moe(72, 2, 2))], residual_mult=0.3),
}


class Case:
    """A model with its checkpoint and plain logits."""

    def __init__(self, path, cfg, seed, steady=True):
        self.cfg, self.w, self.path = cfg, R.weights(cfg, seed, steady), str(path)
        self.rng = np.random.default_rng(seed + 1000)

    def save(self):
        L.write_checkpoint(self.path, R.public(self.cfg), self.w)
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
    most, median = TOL[dt]
    assert np.isfinite(e).all() and e.max() <= factor * most and np.median(e) <= factor * median, (float(e.max()), int(e.argmax()), float(np.median(e)))


# ---- whole models: every shape, prompts, portions, decoding --------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
def test_prompt_portions_and_token_by_token(case, dt):
    toks = case.tokens(200)
    want = case.want(toks)
    eng = mynn.Engine(case.path, dt, 512, prefill_rows=200)
    s = eng.session()
    for sizes in ([200], [1], [2], [3, 1, 31, 2], [33], [64, 65], [170] + [1] * 30):
        close(feed_all(s, toks, sizes), want, dt, 0.4)
        assert s.past_len == len(toks)
        s.reset()
    places = [0, 1, 40, 41, 99, 148]  # only some logits, in gaps
    close(s.feed(toks, places), want[places], dt, 0.4)
    s.close()
    eng.close()


def test_routing_of_the_whole_stream(tmp_path):
    """routers that read what the sublayers write (f32: the choice does not hang on rounding)"""
    cfg = R.config(96, 80, [(R.delta(2, 1, 16, 24), R.moe(48, 6, 2)), (R.parallel(R.window(2, 1, 32, 20), R.memory(2, 8, 8)), R.moe(20, 9, 3))])
    c = Case(tmp_path, cfg, 12, steady=False).save()
    toks = c.tokens(150)
    want = c.want(toks)
    eng = mynn.Engine(c.path, F32, 256)
    s = eng.session()
    for sizes in ([150], [1], [7]):
        close(feed_all(s, toks, sizes), want, F32)
        s.reset()
    s.close()
    eng.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_small_prompt_steps_cut_a_portion(case, dt):
    toks = case.tokens(90)
    eng = mynn.Engine(case.path, dt, 128, prefill_rows=37)
    s = eng.session()
    close(s.feed(toks, list(range(90))), case.want(toks), dt)
    s.close()
    eng.close()


# ---- mechanisms alone -------------------------------------------------------------------------------------------------------
def run_once(path, cfg, w, toks, dt, sizes, max_tokens=512):
    L.write_checkpoint(path, R.public(cfg), w)
    eng = mynn.Engine(str(path), dt, max_tokens)
    s = eng.session()
    got = feed_all(s, toks, sizes)
    s.close()
    eng.close()
    return got


def some_tokens(seed, vocab, n):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


def silence(w, *names):
    for n in names:
        w[n][:] = 0


PLAIN_PARALLEL = R.parallel(R.window(2, 1, 16, 8), R.memory(1, 8, 8))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[40], [1]])
def test_embedding_final_norm_and_head(tmp_path, dt, sizes):
    """a silent mixer: its output is zero, and so is the norm of it"""
    cfg = R.config(80, 60, [(PLAIN_PARALLEL, None)], eps=0.05)
    w = R.weights(cfg, 3)
    silence(w, "l0.mix.left.o", "l0.mix.right.o")
    toks = some_tokens(3, 60, 40)
    want = P.forward(cfg, w, toks)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), want, dt, 0.5)
    plain = dict(w, **{"final.norm": w["final.norm"] - 1.0})  # a weight that is not stored around zero would show
    assert L.row_errors(P.forward(cfg, plain, toks), want).min() > 0.3


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[60], [1], [13]])
@pytest.mark.parametrize("experts,top,ff", [(1, 1, 50), (4, 1, 64), (5, 3, 96), (130, 6, 20), (3, 3, 200)])
def test_experts_alone(tmp_path, dt, sizes, experts, top, ff):
    cfg = R.config(136, 90, [(PLAIN_PARALLEL, R.moe(ff, experts, top))], residual_mult=2.0)
    w = R.weights(cfg, 4)
    silence(w, "l0.mix.left.o", "l0.mix.right.o")
    for e in range(experts):
        w["l0.mlp.e%d.gate" % e] *= 4  # both ends of the activation
    toks = some_tokens(4, 90, 60)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), P.forward(cfg, w, toks), dt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[150], [1], [9]])
@pytest.mark.parametrize("what", ["plain", "slow", "fast", "beta"])
def test_delta_rule_alone(tmp_path, dt, sizes, what):
    cfg = R.config(96, 110, [(R.delta(4, 2, 24, 40, conv=4, ranks=(12, 6)), None)], residual_mult=2.0)
    w = R.weights(cfg, 6)
    if what == "slow":   # nothing decays: the first tokens still count at the end
        w["l0.mix.A_log"][:] = -9.0
    if what == "fast":
        w["l0.mix.A_log"][:] = 2.0
        w["l0.mix.dt_bias"][:] = 0.5
    if what == "beta":
        w["l0.mix.b"] *= 8
    toks = some_tokens(6, 110, 150)
    want = P.forward(cfg, w, toks)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), want, dt)
    if what == "slow":
        assert L.row_errors(P.forward(cfg, w, [toks[0] ^ 1] + toks[1:])[-1:], want[-1:])[0] > 1e-3


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[150], [1], [9], [100, 2]])
@pytest.mark.parametrize("what", ["plain", "remembers", "capped", "small"])
def test_matrix_memory_alone(tmp_path, dt, sizes, what):
    cfg = R.config(96, 110, [(R.parallel(R.window(2, 1, 16, 8), R.memory(3, 24, 40, gate_cap=2.5 if what == "capped" else 12.0)), None)], residual_mult=2.0)
    w = R.weights(cfg, 7)
    silence(w, "l0.mix.left.o")
    if what == "remembers":
        w["l0.mix.right.f.b"][:] = 9.0
    if what == "capped":
        w["l0.mix.right.i"] *= 4
        w["l0.mix.right.f"] *= 4
    if what == "small":      # the normaliser's floor decides
        w["l0.mix.right.i.b"][:] = -6.0
        w["l0.mix.right.k"] *= 0.125
    toks = some_tokens(7, 110, 150)
    want = P.forward(cfg, w, toks)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), want, dt, 2.0)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[300], [1], [9], [250] + [1] * 50])
@pytest.mark.parametrize("left", [
    R.window(4, 2, 32, 48, 3, base=40.0, scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}),   # all three branches
    R.window(3, 1, 40, 1, 0), R.window(2, 2, 24, 1000, 7), R.window(4, 4, 64, 64, 64, conv=7), R.window(8, 1, 20, 65, 200, rot_dims=2)],
    ids=["scaled", "only_itself", "sees_all", "sinks", "long_sinks"])
def test_window_attention_alone(tmp_path, dt, sizes, left):
    cfg = R.config(96, 110, [(R.parallel(left, R.memory(1, 8, 8)), None)], residual_mult=2.0)
    w = R.weights(cfg, 8)
    silence(w, "l0.mix.right.o")
    toks = some_tokens(8, 110, 300)
    close(run_once(tmp_path, cfg, w, toks, dt, sizes), P.forward(cfg, w, toks), dt)


def test_both_scales_count(tmp_path):
    cfg = R.config(64, 70, [(R.parallel(R.window(2, 1, 16, 8), R.memory(2, 8, 12), -0.5, 2.0), None)], residual_mult=-1.5)
    w = R.weights(cfg, 9)
    toks = some_tokens(9, 70, 50)
    want = P.forward(cfg, w, toks)
    for i, sizes in enumerate(([50], [1])):
        close(run_once(tmp_path / str(i), cfg, w, toks, F32, sizes), want, F32)
    for k in ("left_scale", "right_scale"):
        other = json.loads(json.dumps(cfg))
        other["layers"][0]["mixer"][k] = 1.0
        assert L.row_errors(P.forward(other, w, toks), want).max() > 0.1


# ---- kernel forms -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("heads,kv,dim", [(1, 1, 8), (5, 1, 32), (2, 2, 64), (4, 1, 65), (3, 3, 128), (9, 3, 100), (2, 1, 130), (4, 2, 256), (1, 1, 270)])
def test_attention_forms(tmp_path, dt, heads, kv, dim):
    cfg = R.config(64, 64, [(R.parallel(R.window(heads, kv, dim, 150, 10), R.memory(1, 8, 8)), None)], residual_mult=2.0)
    w = R.weights(cfg, heads * 7 + dim)
    silence(w, "l0.mix.right.o")
    toks = some_tokens(dim, 64, 300)
    want = P.forward(cfg, w, toks)
    for i, sizes in enumerate(([300], [270] + [1] * 30, [200, 20, 3, 2])):
        close(run_once(tmp_path / str(i), cfg, w, toks, dt, sizes), want, dt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("heads,kv,dim,vdim", [(1, 1, 4, 5), (3, 1, 33, 7), (2, 2, 64, 130), (2, 1, 128, 128), (4, 2, 150, 20), (1, 1, 256, 64), (2, 1, 300, 24), (1, 1, 512, 9)])
def test_recurrence_forms(tmp_path, dt, heads, kv, dim, vdim):
    """every spread of a state column over lanes, for both recurrences"""
    cfg = R.config(64, 64, [(R.delta(heads, kv, dim, vdim, ranks=(20, 130)), None),
                            (R.parallel(R.window(1, 1, 8, 4), R.memory(heads, dim, vdim)), None)], residual_mult=1.5)
    w = R.weights(cfg, dim)
    silence(w, "l1.mix.left.o")
    toks = some_tokens(dim, 64, 90)
    want = P.forward(cfg, w, toks)
    for i, sizes in enumerate(([90], [60] + [1] * 30, [20, 3, 2])):
        close(run_once(tmp_path / str(i), cfg, w, toks, dt, sizes), want, dt, 2.0)


# ---- one key that decides the answer, at the edges of what a query sees ---------------------------------------------------
class Edges(Case):
    """One attention layer whose queries sit on one key: the query token for a position is searched in the vocabulary."""
    SIZE, KEEP = 70, 4

    def __init__(self, path):
        cfg = R.config(96, 400, [(R.parallel(R.window(4, 2, 48, self.SIZE, self.KEEP, conv=3, rot_dims=4, scale=1.2), R.memory(1, 8, 8)), None)], residual_mult=1.0)
        super().__init__(path, cfg, 21)
        silence(self.w, "l0.mix.right.o")
        # (queries and keys are their own token's projection; the values and the last keys' tails still pass the convolution)
        self.w["l0.mix.left.q.conv"][:] = [0.0, 0.0, 1.0]
        self.w["l0.mix.left.k.conv"][:] = [0.0, 0.0, 1.0]
        self.save()
        self.base = self.tokens(400)

    def query_for(self, n, p):
        """(tokens of n positions whose last one looks at position p, its softmax weight there were everything visible)"""
        c, m = self.cfg, self.cfg["layers"][0]["mixer"]["left"]
        toks = self.base[:n]
        _, k, _ = P.attention_parts(self.w["embed"][toks], self.w, "l0.mix.left.", m, c["norm"]["eps"])
        q = P.rms(self.w["embed"] @ self.w["l0.mix.left.q"].T, c["norm"]["eps"]) * self.w["l0.mix.left.q.norm"]
        q = q.reshape(-1, 4, 48)
        freq = P.rotary_frequencies(m["rot"])
        for i, f in enumerate(freq):
            co, si, u, v = np.cos((n - 1) * f), np.sin((n - 1) * f), q[..., 2 * i].copy(), q[..., 2 * i + 1].copy()
            q[..., 2 * i], q[..., 2 * i + 1] = u * co - v * si, v * co + u * si
        s = np.einsum("vhd,khd->vhk", q, np.repeat(k[:n - 1], 2, axis=1)) * m["scale"]
        lead = s[:, :, p] - np.delete(s, p, axis=2).max(-1)
        best = int(np.unravel_index(lead.argmax(), lead.shape)[0])
        return toks[:n - 1] + [best], float(lead.max())


@pytest.fixture(scope="module")
def edges(tmp_path_factory):
    return Edges(tmp_path_factory.mktemp("edges"))


@pytest.mark.parametrize("dt", DTYPES)
def test_keys_at_the_edges_of_a_window(edges, dt):
    """just inside and just outside the window and the kept tokens, at page borders, near, in prompts and decoded; a window
    or a count of kept tokens that is one off in the statement gives another answer"""
    c, size, keep = edges, edges.SIZE, edges.KEEP
    eng = mynn.Engine(c.path, dt, 512, prefill_rows=400)
    s = eng.session()
    tried, shown = 0, {"size-1": 0, "size+1": 0, "keep-1": 0, "keep+1": 0}
    for n in (80, 129, 135, 193, 300, 391):
        for p in {n - size, n - size - 1, keep - 1, keep, 0, n - 2, 63, 64, 127, 128, 255, 256}:
            if not 0 <= p < n - 1:
                continue
            toks, lead = c.query_for(n, p)
            if lead < 1.0:
                continue
            tried += 1
            want = c.want(toks)[-1:]
            for sizes in ([n], [n - 1, 1], [n - 2, 2], [n - 40, 40]):
                at = 0
                for m in sizes:
                    got = s.feed(toks[at:at + m], [m - 1])
                    at += m
                s.reset()
                close(got, want, dt, 4.0)
            for name, key, by in (("size-1", "size", -1), ("size+1", "size", 1), ("keep-1", "keep_first", -1), ("keep+1", "keep_first", 1)):
                if p != {"size-1": n - size, "size+1": n - size - 1, "keep-1": keep - 1, "keep+1": keep}[name] or (key == "keep_first" and n <= size + keep):
                    continue
                other = json.loads(json.dumps(c.cfg))
                other["layers"][0]["mixer"]["left"]["mask"][key] += by
                shown[name] += L.row_errors(P.forward(other, c.w, toks)[-1:], want)[0] > 0.2
    assert tried >= 30 and min(shown.values()) >= 3, (tried, shown)
    s.close()
    eng.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_first_tokens_and_convolution_tails(tmp_path, dt):
    """each of the first tokens alone in its portion, and portions shorter than the convolutions' reach"""
    cfg = R.config(64, 90, [(R.delta(2, 1, 16, 16, conv=6), None), (R.parallel(R.window(2, 1, 16, 3, 1, conv=8), R.memory(1, 8, 8)), None)], residual_mult=1.0)
    c = Case(tmp_path, cfg, 31)
    for t in ("l0.mix.q.conv", "l0.mix.k.conv", "l0.mix.v.conv", "l1.mix.left.q.conv", "l1.mix.left.k.conv"):
        c.w[t][:, 0] = 1.5  # the oldest input counts
    c.save()
    toks = c.tokens(40)
    want = c.want(toks)
    eng = mynn.Engine(c.path, dt, 128)
    s = eng.session()
    for sizes in ([1], [2], [3, 2], [5, 1, 2, 4], [1, 2, 3, 4, 5, 6, 7]):
        close(feed_all(s, toks, sizes), want, dt, 1.5)
        s.reset()
    s.close()
    eng.close()


# ---- cache and state: pages, slots, sessions, reuse ---------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
def test_sessions_share_pages_and_reuse_states(case, dt):
    """Two sessions grow in turns over one pool; one ends, and its pages and its states serve a third.  The logits do not depend
    on which pages and states a session holds (bit for bit), nor on what was there before."""
    a, b, c = case.tokens(140), case.tokens(75), case.tokens(200)
    eng = mynn.Engine(case.path, dt, 448, max_seq=256, prefill_rows=64)
    free0 = eng.free_rows
    one = eng.session()
    alone = {}
    for name, toks, sizes in (("a", a, [50, 3, 1, 1]), ("b", b, [30, 1]), ("c", c, [64, 1, 1, 2])):
        alone[name] = feed_all(one, toks, sizes)
        one.reset()
    assert eng.free_rows == free0
    two = eng.session()
    got_a, got_b, ia, ib, i = [], [], 0, 0, 0
    while ia < len(a) or ib < len(b):
        n, m = [50, 3, 1, 1][i % 4], [30, 1][i % 2]
        if ia < len(a):
            n = min(n, len(a) - ia)
            got_a.append(one.feed(a[ia:ia + n], list(range(n))))
            ia += n
        if ib < len(b):
            m = min(m, len(b) - ib)
            got_b.append(two.feed(b[ib:ib + m], list(range(m))))
            ib += m
        i += 1
    assert np.array_equal(np.concatenate(got_a), alone["a"]) and np.array_equal(np.concatenate(got_b), alone["b"])
    close(alone["a"], case.want(a), dt)
    one.close()                       # its pages and its states go to the next session
    three = eng.session()
    got_c = feed_all(three, c, [64, 1, 1, 2])
    assert np.array_equal(got_c, alone["c"])
    close(got_c, case.want(c), dt)
    close(feed_all(two, b[:1], [1]), case.want(b + b[:1])[-1:], dt)  # the other one goes on unharmed
    for s in (two, three):
        s.close()
    assert eng.free_rows == free0
    eng.close()


def test_a_state_cannot_go_back(tmp_path):
    c = Case(tmp_path, MODELS["mixed"], 3).save()
    toks = c.tokens(60)
    eng = mynn.Engine(c.path, F32, 128)
    s = eng.session()
    s.feed(toks, [])
    s.past_len = 40
    with pytest.raises(mynn.MynnError, match="sequence state"):
        s.feed(toks[:2], [1])
    with pytest.raises(mynn.MynnError):
        s.generate_ids(toks[:2], 3)
    s.past_len = 60
    close(s.feed(toks[:5], [4]), c.want(toks + toks[:5])[-1:], F32)
    s.past_len = 0                    # from the start is always possible
    close(s.feed(toks[:9], [8]), c.want(toks[:9])[-1:], F32)
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
    """state memory full of NaN: a sequence's first step reads none of it"""
    arch = mynn.Arch(case.path)
    w = device_weights(case, dt)
    B, N, D = 3, 70, 6
    seqs = [case.tokens(N + D) for _ in range(B)]
    pool = pages = None
    if paged:
        pool = mynn.KvPool(B * 2 + 3, 64)
        pages = mynn.KvPages(pool, B, 128)
        state = mynn.layered_state(arch, dt, pool.n_pages * 64, fill=0xFF, batch=B)
    else:
        state = mynn.layered_state(arch, dt, B * 128, fill=0xFF, batch=B)
    pre = mynn.LayeredDecoder(arch, w, dt, 128, seq_q=64, batch=B, state=state, kv_pages=pages)
    dec = mynn.LayeredDecoder(arch, w, dt, 128, batch=B, state=state, kv_pages=pages)
    for cuts in ([0, 40, 60, N], [0, 1, 3, N - 1, N]):
        got = [[] for _ in range(B)]
        for lo, hi in zip(cuts, cuts[1:]):
            for at in range(lo, hi, 64):
                m = min(64, hi - at)
                _, lg = (pre if m > 1 else dec).step_rows([s[at:at + m] for s in seqs], m, at, n_logits=m)
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
    c = Case(tmp_path, MODELS["mixed"], 2).save()
    arch = mynn.Arch(c.path)
    dec = mynn.LayeredDecoder(arch, device_weights(c, BF16), BF16, 128)
    # embedding; delta rule 3 + experts 3; attention and memory 4 (the second one's keys come in two ranges: + 1), experts 3; head, token
    assert dec.stats() == dict(dec.stats(), launches_per_step=1 + 6 + 4 + 5 + 3 + 2, graph=True)
    names = [n for n, ms, _, _ in dec.profile_step(3, 0) if ms > 0]
    assert names.count("delta_step") == 1 and names.count("window_attention") == 2 and names.count("gemv_router") == 2 and names[-1] == "greedy_advance"
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
    # a second turn continues the same sequence
    assert s.generate_ids([ids[-1], 5], 3) == plain_greedy(case, prompt + ids + [5], 3)[0]
    s.close()
    # an end-of-sequence id inside a run of the device loop: what the run read past it must not be in the states
    stop = ids[9]
    s = eng.session(eos=stop)
    cut = ids[:ids.index(stop) + 1]
    assert s.generate_ids(prompt, 40) == cut
    assert s.past_len == len(prompt) + len(cut) - 1
    close(s.feed([cut[-1], 7, 3], [0, 1, 2]), case.want(prompt + cut + [7, 3])[-3:], F32)
    s.close()
    eng.close()


def test_long_decoding_in_graph_runs_matches_the_prompt_path(tmp_path):
    """300 tokens from the device-resident loop; the same tokens fed as a prompt must name every one of them"""
    c = Case(tmp_path, MODELS["mixed"], 31).save()
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
        close(lg, c.want(prompt + ids[:-1])[9:], dt)
        s.close()
        eng.close()


# ---- the trace program ------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,dt", [("float32", F32), ("bfloat16", BF16)])
def test_trace_program(case, tmp_path, dtype, dt):
    a, b = case.tokens(90), case.tokens(40)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:60], "want": [59, 0, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[60:62], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[62:63], "want": [0]}], "end": []},
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
