// Executor of decoders described layer by layer (ModelSpec): a 32-bit residual stream, layers with norms behind (and, if the
// description says so, in front of) their sublayers, whose mixer and feed-forward come from the description, and layer ranges
// that run several times.  It fills the executor's build and
// enqueue hooks; inputs, pages, graph capture, the device-resident loop, profile and session are decoder.hip's and
// llm_session.hip's, the same as for the Llama graph.
//
// Session state: a cache per layer run with attention (a looped layer has one per pass), [batch, max_seq, row] or pages of it,
// then the token history [batch, max_seq] int32 in the same rows: a pair embedding reads a step's previous token there, so it
// is found again after a rewind, in any portion and on any page.  Runs with a recurrence or a short convolution have a block
// per sequence behind these, which a step from position 0 starts afresh.
//
// One new token (decode, batch 1): per run the input projection [norms and residual sum in its prologue], latent_prepare,
// attention, merge + W_uv + gate, output projection, gate/up, down -- 7 launches; all scalars in device memory, captured
// into the decode graphs.  More rows: the same with one residual_norm_rows pass per norm and matrix-core products.
#include <algorithm>
#include <cmath>

#include "layered.h"

namespace mynn {

void layered_weights_free(LayeredWeights *w) {
    if (!w) return;
    for (void *p : w->owned) (void)hipFree(p);
    delete w;
}

// portions up to this many rows take the absorbed attention (its work grows with the latent's width per query, the
// expanded form's with the number of keys it has to expand)
constexpr int kAbsorbRows = 32;

void destroy_layered(Model &m) {
    for (void *p : m.net->rot_tables) (void)hipFree(p);
    if (m.net->saved) (void)hipFree(m.net->saved);
    delete m.net;
    m.net = nullptr;
}

// ---- padded weight copies, once per weight set ------------------------------------------------------------------------
int WeightPacker::alloc(void **p, size_t rows, size_t cols, size_t elem) {
    const size_t bytes = rows * cols * (elem ? elem : dtype_size(dt));
    MYNN_HIP(hipMalloc(p, bytes));
    w.owned.push_back(*p);
    m.wset->bytes_repack += bytes;
    MYNN_HIP(hipMemsetAsync(*p, 0, bytes, m.stream));
    return 0;
}
int WeightPacker::vec(void **p, const std::string &name, int heads, int n, int np, int padded) {
    TRY(alloc(p, 1, padded));
    return pack_blocks(PackBlocks{*p, src(name), padded, (long)heads * n, 1, 1, 0, 1, 0, 1, heads, n, 0, np, n, 0, 0}, dt, m.stream);
}
int WeightPacker::rows(DenseW &l, const std::string &name, int heads, int n, int np, int row0) {
    return pack_blocks(PackBlocks{l.w, src(name), l.K, s.width, heads, n, row0, np, 0, n, 1, s.width, 0, s.width, s.width, 0, 0}, dt, m.stream);
}
int WeightPacker::cols(DenseW &l, const std::string &name, int heads, int n, int np, int col0) {
    return pack_blocks(PackBlocks{l.w, src(name), l.K, (long)heads * n, 1, s.width, 0, s.width, 0, s.width, heads, n, col0, np, n, 0, 0}, dt, m.stream);
}

static int pack_latent(WeightPacker &pk, LayerWeights &o, const MixerSpec &mix, const std::string &mx) {
    const int W = pk.s.width, ld = pk.ld;
    const LatentDims d = latent_dims(mix);
    TRY(pk.norm(&o.latent_norm, mx + "dkv.norm", d.rank, d.rp));
    // input projection: q head by head [dim | rotated], latent, rotated key part, gates
    TRY(pk.linear(o.in, d.n_in(), ld));
    auto in_rows = [&](const char *t, int H, int rows, int dst0, int dst_rs, int src0, int src_rs) {
        return pack_blocks(PackBlocks{o.in.w, pk.src(mx + t), ld, W, H, rows, dst0, dst_rs, src0, src_rs, 1, W, 0, W, W, 0, 0}, pk.dt, pk.m.stream);
    };
    TRY(in_rows("q", d.H, d.dim, 0, d.dk(), 0, d.dim + d.rot));
    TRY(in_rows("q", d.H, d.rot, d.dimp, d.dk(), d.dim, d.dim + d.rot));
    TRY(in_rows("dkv", 1, d.rank, d.qcols(), 1, 0, 1));
    TRY(in_rows("dkv", 1, d.rot, d.qcols() + d.rp, 1, d.rank, 1));
    TRY(in_rows("g", 1, d.H, d.qcols() + d.lw(), 1, 0, 1));
    // key rows of every head, then value rows
    TRY(pk.linear(o.ukv, d.kvcols(), d.rp));
    TRY(pack_blocks(PackBlocks{o.ukv.w, pk.src(mx + "uk"), d.rp, d.rank, d.H, d.dim, 0, d.dimp, 0, d.dim, 1, d.rank, 0, d.rank, d.rank, 0, 0}, pk.dt, pk.m.stream));
    TRY(pack_blocks(PackBlocks{o.ukv.w, pk.src(mx + "uv"), d.rp, d.rank, d.H, d.vdim, d.H * d.dimp, d.vdimp, 0, d.vdim, 1, d.rank, 0, d.rank, d.rank, 0, 0}, pk.dt, pk.m.stream));
    TRY(pk.linear(o.o, ld, d.acols()));
    TRY(pack_blocks(PackBlocks{o.o.w, pk.src(mx + "o"), d.acols(), (long)d.H * d.vdim, 1, W, 0, W, 0, W, d.H, d.vdim, 0, d.vdimp, d.vdim, 0, 0}, pk.dt, pk.m.stream));
    return 0;
}

static int make_weights(Model &m, const ModelSpec &s) {
    WeightSet &ws = *m.wset;
    if (ws.layered && ws.layered->ready) return 0;
    layered_weights_free(ws.layered);
    ws.layered = new LayeredWeights;
    LayeredWeights &w = *ws.layered;
    const int dt = m.cfg.dtype, W = s.width, ld = pad_to(W, 64);
    ws.bytes_repack = 0;
    WeightPacker pk{m, w, s, dt, ld};
    for (size_t i = 0; i < s.tensors.size(); i++)
        MYNN_REQUIRE(ws.initializer[i], MYNN_ERR_INVALID, "model_init: null weight %s", s.tensors[i].name.c_str());
    auto src = [&](const std::string &name) { return pk.src(name); };
    auto norm = [&](void **p, const std::string &name, int n, int padded) { return pk.norm(p, name, n, padded); };
    auto linear = [&](DenseW &l, int N, int K) { return pk.linear(l, N, K); };
    w.layers.resize(s.layers.size());
    for (size_t i = 0; i < s.layers.size(); i++) {
        const LayerSpec &L = s.layers[i];
        const std::string p = "l" + std::to_string(i) + ".", mx = p + "mix.";
        LayerWeights &o = w.layers[i];
        if (s.pre_norm) TRY(norm(&o.norm1, p + "norm1", W, ld));
        TRY(norm(&o.norm1b, p + (s.pre_norm ? "norm1b" : "norm1"), W, ld));
        if (L.mlp.kind != MlpSpec::NONE) {
            if (s.pre_norm) TRY(norm(&o.norm2, p + "norm2", W, ld));
            TRY(norm(&o.norm2b, p + (s.pre_norm ? "norm2b" : "norm2"), W, ld));
        }
        if (L.mlp.kind == MlpSpec::EXPERTS) TRY(pack_experts(pk, o, L.mlp, p + "mlp."));
        if (L.mixer.kind == MixerSpec::PARALLEL) TRY(pack_parallel(pk, o, L.mixer, mx));
        if (L.mixer.kind == MixerSpec::CHANNEL_DELTA) TRY(pack_channel_delta(pk, o, L.mixer, mx));
        if (L.mixer.kind == MixerSpec::LATENT_ATTENTION) TRY(pack_latent(pk, o, L.mixer, mx));
        if (L.mlp.kind != MlpSpec::GATED_DENSE) continue;
        const int F = L.mlp.ff, Fp = pad_to(F, 64);
        TRY(linear(o.gu, 2 * Fp, ld));
        TRY(pack_blocks(PackBlocks{o.gu.w, src(p + "mlp.gate"), ld, W, 1, F, 0, F, 0, F, 1, W, 0, W, W, 32, 0}, dt, m.stream));
        TRY(pack_blocks(PackBlocks{o.gu.w, src(p + "mlp.up"), ld, W, 1, F, 0, F, 0, F, 1, W, 0, W, W, 32, 1}, dt, m.stream));
        TRY(linear(o.down, ld, Fp));
        TRY(pack_blocks(PackBlocks{o.down.w, src(p + "mlp.down"), Fp, F, 1, W, 0, W, 0, W, 1, F, 0, F, F, 0, 0}, dt, m.stream));
    }
    if (s.loop.times) {
        TRY(linear(w.loop_in, ld, 2 * ld));
        TRY(pack_blocks(PackBlocks{w.loop_in.w, src("loop.in"), 2L * ld, 2L * W, 1, W, 0, W, 0, W, 2, W, 0, ld, W, 0, 0}, dt, m.stream));
    }
    TRY(norm(&w.final_norm, "final.norm", W, ld));
    TRY(linear(w.head, s.vocab, ld));
    TRY(pack_blocks(PackBlocks{w.head.w, src("head"), ld, W, 1, s.vocab, 0, s.vocab, 0, s.vocab, 1, W, 0, W, W, 0, 0}, dt, m.stream));
    MYNN_HIP(hipStreamSynchronize(m.stream));
    w.ready = true;
    return 0;
}

// (cos, sin) of every position, angles in double, one table per distinct rotation
static int make_rotary_tables(LayeredNet &n, int max_seq) {
    const ModelSpec &s = *n.spec;
    n.rot.assign(s.layers.size(), nullptr);
    auto rotary = [&](size_t i) -> const RotarySpec & {
        const MixerSpec &m = s.layers[i].mixer;
        return m.kind == MixerSpec::PARALLEL ? m.window.rot : m.rot;
    };
    for (size_t i = 0; i < s.layers.size(); i++) {
        const RotarySpec &r = rotary(i);
        if (!r.dims) continue;
        for (size_t j = 0; j < i && !n.rot[i]; j++)
            if (rotary(j) == r) n.rot[i] = n.rot[j];
        if (n.rot[i]) continue;
        const int half = r.dims / 2;
        std::vector<float2> t((size_t)max_seq * half);
        for (int k = 0; k < half; k++) {
            const double f = r.frequency(k);
            for (int p = 0; p < max_seq; p++) t[(size_t)p * half + k] = float2{(float)cos(p * f), (float)sin(p * f)};
        }
        void *d = nullptr;
        MYNN_HIP(hipMalloc(&d, t.size() * sizeof(float2)));
        n.rot_tables.push_back(d);
        MYNN_HIP(hipMemcpy(d, t.data(), t.size() * sizeof(float2), hipMemcpyHostToDevice));
        n.rot[i] = (float2 *)d;
    }
    return 0;
}

int build_layered(Model &m, void **state) {
    const mynn_model_config &c = m.cfg;
    m.net = new LayeredNet;
    LayeredNet &n = *m.net;
    n.spec = arch_spec(c.arch);
    const ModelSpec &s = *n.spec;
    MYNN_HIP(hipStreamCreateWithFlags(&m.stream, hipStreamNonBlocking));
    {
        std::lock_guard<std::mutex> lk(m.wset->mu);
        TRY(make_weights(m, s));
        n.w = m.wset->layered;
        n.embed = m.wset->initializer[s.tensor_index("embed")];
        if (s.bigram.buckets) n.bigram = m.wset->initializer[s.tensor_index("bigram")];
    }
    TRY(make_rotary_tables(n, c.max_seq));
    for (size_t i = 0; i < s.states.size(); i++)
        MYNN_REQUIRE(state[i] && ((int)i == s.history || aligned16(state[i])), MYNN_ERR_INVALID, "model_init: null or misaligned state buffer %zu", i);
    for (const LayerRun &r : s.runs) {
        n.caches.push_back(r.cache < 0 ? nullptr : state[r.cache]);
        n.memory.push_back(r.memory < 0 ? nullptr : (float *)state[r.memory]);
    }
    n.history = (int32_t *)state[s.history];
    if (c.kv_page_rows) {
        m.pages = (mynn_kv_pages *)state[s.states.size()];
        TRY(executor_bind_pages(m));
    }

    const int rows = c.batch * c.seq_q, ld = n.ld = pad_to(s.width, 64);
    const size_t eb = dtype_size(c.dtype);
    const int abs_rows = std::min(c.seq_q, kAbsorbRows);
    MixerScratch sc;
    size_t q_abs = 0, c_rows = 0, rot_rows = 0, kv = 0;
    n.gemv = dense_gemv_supported(ld) && (!s.loop.times || dense_gemv_supported(2 * ld));
    for (const LayerSpec &L : s.layers) {
        TRY(check_mixer(L.mixer));
        int acols = 0;
        if (L.mixer.kind == MixerSpec::LATENT_ATTENTION) {
            const LatentDims d = latent_dims(L.mixer);
            sc.proj = std::max<size_t>(sc.proj, (size_t)rows * d.n_in() * eb);
            acols = d.acols();
            const bool expanded = latent_expanded_supported(d, c.dtype);
            const size_t absorbed = (size_t)c.batch * (expanded ? abs_rows : c.seq_q);
            size_t parts = 0;  // (row, head) x ranges of any portion
            for (int S = 1; S <= (expanded ? abs_rows : c.seq_q); S++)
                parts = std::max(parts, (size_t)c.batch * S * d.H * latent_absorbed_splits(c.batch, S, d, c.max_seq, c.dtype));
            q_abs = std::max(q_abs, absorbed * d.H * d.lw());
            sc.part_o = std::max(sc.part_o, parts * d.rp * 4);
            sc.part_ml = std::max(sc.part_ml, parts * 2 * 4);
            if (expanded && c.seq_q > kAbsorbRows) {
                c_rows = std::max(c_rows, (size_t)c.max_seq * d.rp);
                rot_rows = std::max(rot_rows, (size_t)c.max_seq * d.rotp);
                kv = std::max(kv, (size_t)c.max_seq * d.kvcols());
            }
        } else {
            scratch_recurrent(sc, L.mixer, c);
            acols = L.mixer.kind == MixerSpec::PARALLEL ? parallel_dims(L.mixer).acols() : delta_dims(L.mixer.delta).acols();
        }
        sc.attn = std::max(sc.attn, (size_t)rows * acols * eb);
        const int fp = pad_to(L.mlp.ff, 64);
        n.gemv = n.gemv && dense_gemv_supported(acols);
        if (L.mlp.kind == MlpSpec::GATED_DENSE) {
            sc.hmid = std::max(sc.hmid, (size_t)rows * fp * eb);
            n.gemv = n.gemv && dense_gemv_supported(fp);
        }
        if (L.mlp.kind == MlpSpec::EXPERTS) {
            scratch_experts(sc, L.mlp, c, ld);
            n.gemv = n.gemv && expert_row_supported(ld, fp, L.mlp.top);
        }
    }
    m.token_cap = c.max_seq + 8;
    ArenaPlan plan;
    const size_t o_xa = plan.take((size_t)rows * ld * 4), o_xb = plan.take((size_t)rows * ld * 4);
    const size_t o_x0 = plan.take(s.loop.times ? (size_t)rows * ld * 4 : 0);
    const size_t o_act = plan.take((size_t)rows * ld * (s.loop.times ? 2 : 1) * eb), o_proj = plan.take(sc.proj);
    const size_t o_attn = plan.take(sc.attn), o_y = plan.take((size_t)rows * ld * eb), o_h = plan.take(sc.hmid);
    const size_t o_qa = plan.take(q_abs * eb), o_po = plan.take(sc.part_o), o_pm = plan.take(sc.part_ml);
    const size_t o_c = plan.take(c_rows * eb), o_r = plan.take(rot_rows * eb), o_kv = plan.take(kv * eb);
    const size_t o_l = plan.take((size_t)rows * s.vocab * 4), o_sc = plan.take(32 + (size_t)c.batch * 4);
    const size_t o_ids = plan.take((size_t)rows * 8), o_pos = plan.take((size_t)c.seq_q * 8), o_tok = plan.take((size_t)m.token_cap * 4);
    const size_t o_q = plan.take(sc.q), o_low = plan.take(sc.low), o_gates = plan.take(sc.gates), o_o = plan.take(sc.o), o_qk = plan.take(sc.qk);
    const size_t o_v = plan.take(sc.v), o_beta = plan.take(sc.beta), o_bl = plan.take(sc.blocks), o_dec = plan.take(sc.dec), o_rt = plan.take(sc.router), o_score = plan.take(sc.score);
    const size_t o_parts = plan.take(sc.parts), o_chosen = plan.take(sc.chosen), o_choice = plan.take(sc.choice), o_tg = plan.take(sc.tile_group);
    const size_t o_slot = plan.take(sc.slot), o_hs = plan.take(sc.hsort);
    const size_t o_ls = plan.take(4), o_cand = plan.take(kGreedyCands * sizeof(GreedyCand));
    m.arena_bytes = plan.off;
    MYNN_HIP(hipMalloc((void **)&m.arena, m.arena_bytes));
    MYNN_HIP(hipMemset(m.arena, 0, m.arena_bytes));
    n.xa = (float *)(m.arena + o_xa); n.xb = (float *)(m.arena + o_xb); n.x0 = s.loop.times ? (float *)(m.arena + o_x0) : nullptr;
    n.act = m.arena + o_act; n.proj = m.arena + o_proj; n.attn = m.arena + o_attn; n.y = m.arena + o_y; n.hmid = m.arena + o_h;
    n.q_abs = m.arena + o_qa; n.part_o = (float *)(m.arena + o_po); n.part_ml = (float *)(m.arena + o_pm);
    n.c_rows = m.arena + o_c; n.rot_rows = m.arena + o_r; n.kv = m.arena + o_kv;
    n.q = m.arena + o_q; n.low = m.arena + o_low; n.gates = (float *)(m.arena + o_gates); n.o = (float *)(m.arena + o_o); n.qk = (float *)(m.arena + o_qk);
    n.v = (float *)(m.arena + o_v); n.beta = (float *)(m.arena + o_beta); n.blocks = (float *)(m.arena + o_bl); n.dec = (float *)(m.arena + o_dec); n.router = (float *)(m.arena + o_rt);
    n.score = (float *)(m.arena + o_score); n.parts = (float *)(m.arena + o_parts); n.chosen = (int32_t *)(m.arena + o_chosen);
    n.choice = (int32_t *)(m.arena + o_choice); n.tile_group = (int32_t *)(m.arena + o_tg); n.slot = (int32_t *)(m.arena + o_slot); n.hsort = m.arena + o_hs;
    m.logits = m.arena + o_l;
    m.d_past = (int32_t *)(m.arena + o_sc); m.d_active = m.d_past + 1; m.d_step = m.d_past + 2; m.d_next = m.d_past + 8;
    m.d_ids = (int64_t *)(m.arena + o_ids); m.d_pos = (int64_t *)(m.arena + o_pos); m.d_tokens = (int32_t *)(m.arena + o_tok);
    n.logit_scale = (float *)(m.arena + o_ls);
    n.cand = (GreedyCand *)(m.arena + o_cand);
    MYNN_HIP(hipMemcpy(n.logit_scale, &s.logit_scale, 4, hipMemcpyHostToDevice));
    m.next_stage = align_up((size_t)c.batch * 4, 256);
    m.stage_bytes = align_up((size_t)rows * 8 + (size_t)c.seq_q * 8 + 64 + (size_t)m.token_cap * 4, 256) + 256 + m.next_stage;
    MYNN_HIP(hipHostMalloc((void **)&m.h_stage, m.stage_bytes, hipHostMallocDefault));
    MYNN_HIP(hipDeviceSynchronize());
    return 0;
}

// ---- one step -------------------------------------------------------------------------------------------------------------
int linear(Stream &s, void *out, const DenseW &w, int store, const char *name, const char *gemv_name, const void *act, const void *wa, int pro) {
    const int dt = s.m.cfg.dtype;
    const double eb = dtype_size(dt), ob = store == DENSE_F32 ? 4 : eb, n_out = store == DENSE_GEGLU ? w.N / 2 : w.N;
    if (s.one) {
        ResidualNorm r = s.row(wa);
        note(s.m, gemv_name, (double)w.N * w.K * eb + (pro == PRO_ROWS ? w.K * eb : s.row_bytes(eb)) + n_out * ob, 2.0 * w.N * w.K);
        TRY(dense_gemv(out, act, pro == PRO_ROWS ? nullptr : &r, pro, w.w, w.N, w.K, store, nullptr, dt, s.m.stream));
        if (pro != PRO_ROWS) s.added();
        return 0;
    }
    if (pro != PRO_ROWS) {
        note(s.m, "residual_norm", s.rows * (s.row_bytes(eb) + s.n.ld * eb * (pro == PRO_RESIDUAL_CONCAT ? 2 : 1)));
        TRY(residual_norm_rows(s.n.act, s.row(wa), pro, 0, 1, s.rows, dt, s.m.stream));
        s.added();
        act = s.n.act;
    }
    note(s.m, name, ((double)w.N * w.K + (double)s.rows * w.K) * eb + s.rows * n_out * ob, 2.0 * s.rows * w.N * w.K);
    return dense_gemm(out, act, w.w, s.rows, w.N, w.K, store, nullptr, dt, s.m.stream);
}

namespace {
// ---- latent attention: acts on n.proj / n.attn, leaves the sublayer output in n.y
int latent_attention(Stream &st, int run, const LayerWeights &w, const MixerSpec &mix) {
    Model &m = st.m;
    LayeredNet &n = st.n;
    const mynn_model_config &c = m.cfg;
    const LatentDims d = latent_dims(mix);
    const double eb = dtype_size(c.dtype);
    const int S = m.rows_now, B = c.batch;
    TRY(linear(st, n.proj, w.in, DENSE_T, "linear_latent_in", "gemv_norm_latent_in", nullptr, w.norm1, PRO_RESIDUAL_NORM));
    LatentParams p{};
    p.d = d; p.scale = mix.scale; p.eps = n.spec->eps; p.rot_dims = mix.rot.dims; p.rot = n.rot[n.spec->runs[run].layer];
    p.proj = n.proj; p.norm_w = w.latent_norm; p.ukv = w.ukv.w; p.cache = n.caches[run]; p.paging = m.paging;
    p.d_past = m.d_past; p.B = B; p.S = S; p.max_seq = c.max_seq; p.out = n.attn;
    p.q_abs = n.q_abs; p.part_o = n.part_o; p.part_ml = n.part_ml;
    p.c_rows = n.c_rows; p.rot_rows = n.rot_rows; p.kv = n.kv;
    const bool absorb = S <= kAbsorbRows || !latent_expanded_supported(d, c.dtype);
    note(m, absorb ? "latent_absorb_append" : "latent_rotate_append",
         absorb ? (double)d.H * d.dim * d.rp * eb + st.rows * (d.n_in() + d.H * d.lw() + d.lw()) * eb : st.rows * (2.0 * d.lw() + 2.0 * d.H * d.rot) * eb,
         absorb ? 2.0 * st.rows * d.H * d.dim * d.rank : 0.0);
    TRY(latent_prepare(p, absorb, c.dtype, m.stream));
    if (absorb) {
        p.nsplit = latent_absorbed_splits(B, S, d, c.max_seq, c.dtype);
        // (bytes: queries only; the cache rows read depend on the context, which the host does not know under replay)
        note(m, "latent_attention", (double)st.rows * d.H * d.lw() * eb);
        TRY(latent_attention_absorbed(p, c.dtype, m.stream));
        note(m, "latent_merge_out", (double)d.H * d.vdim * d.rp * eb + (double)st.rows * d.H * (d.rp * 4 + d.vdimp * eb), 2.0 * st.rows * d.H * d.vdim * d.rank);
        TRY(latent_merge_out(p, c.dtype, m.stream));
    } else {
        const int L = m.h_past + S;
        for (int b = 0; b < B; b++) {
            // (one sequence: latent_prepare has put the new tokens' rows in place already)
            const int gather = B == 1 ? m.h_past : L;
            if (gather) {
                note(m, "latent_gather", 2.0 * gather * d.lw() * eb);
                TRY(latent_gather(p, b, gather, c.dtype, m.stream));
            }
            note(m, "linear_latent_kv", ((double)L * d.rp + (double)w.ukv.N * w.ukv.K + (double)L * w.ukv.N) * eb, 2.0 * L * w.ukv.N * w.ukv.K);
            TRY(dense_gemm(n.kv, n.c_rows, w.ukv.w, L, w.ukv.N, w.ukv.K, DENSE_T, nullptr, c.dtype, m.stream));
            note(m, "latent_attention", (double)(S * (d.qcols() + d.acols()) + L * (d.kvcols() + d.rotp)) * eb,
                 2.0 * d.H * (d.dim + d.rot + d.vdim) * ((double)S * m.h_past + 0.5 * S * (S + 1.0)));
            TRY(latent_attention_expanded(p, b, m.h_past, c.dtype, m.stream));
        }
    }
    return linear(st, n.y, w.o, DENSE_T, "linear_o", "gemv_o", n.attn, nullptr, PRO_ROWS);
}
}  // namespace

int enqueue_layered(Model &m) {
    LayeredNet &n = *m.net;
    const ModelSpec &s = *n.spec;
    const mynn_model_config &c = m.cfg;
    const int dt = c.dtype, S = m.rows_now, rows = c.batch * S;
    const double eb = dtype_size(dt);
    m.record.clear();
    for (hipEvent_t e : m.events) hipEventDestroy(e);
    m.events.clear();

    note(m, "embed", (double)rows * (s.width * eb * (s.bigram.buckets ? 2 : 1) + n.ld * 4.0 * (n.x0 ? 2 : 1)));
    TRY(embed_tokens(EmbedParams{n.xa, n.x0, n.embed, n.bigram, s.bigram.buckets, s.bigram.mul_prev, s.bigram.mul_cur, m.d_ids, m.d_past,
                                 n.history, m.paging, c.batch, S, s.width, n.ld, s.vocab, c.max_seq}, dt, m.stream));
    Stream st{m, n, rows, rows == 1 && n.gemv, n.xa, n.xb};
    for (size_t r = 0; r < s.runs.size(); r++) {
        const LayerSpec &L = s.layers[s.runs[r].layer];
        const LayerWeights &w = n.w->layers[s.runs[r].layer];
        if (s.runs[r].starts_pass) {
            // x <- W_in [x + what is still to be added; x0]: the sum itself is read by this linear only
            ResidualNorm row = st.row(nullptr);
            row.x_out = nullptr;
            if (st.one) {
                note(m, "gemv_loop_in", (double)n.w->loop_in.N * n.w->loop_in.K * eb + st.row_bytes(eb) + n.ld * 8.0, 2.0 * n.w->loop_in.N * n.w->loop_in.K);
                TRY(dense_gemv(st.other, nullptr, &row, PRO_RESIDUAL_CONCAT, n.w->loop_in.w, n.ld, 2 * n.ld, DENSE_F32, nullptr, dt, m.stream));
            } else {
                note(m, "residual_concat", rows * (st.row_bytes(eb) + n.ld * (4 + 2 * eb)));
                TRY(residual_norm_rows(n.act, row, PRO_RESIDUAL_CONCAT, 0, 1, rows, dt, m.stream));
                note(m, "linear_loop_in", (double)(n.w->loop_in.N + rows) * n.w->loop_in.K * eb + rows * n.ld * 4.0, 2.0 * rows * n.w->loop_in.N * n.w->loop_in.K);
                TRY(dense_gemm(st.other, n.act, n.w->loop_in.w, rows, n.ld, 2 * n.ld, DENSE_F32, nullptr, dt, m.stream));
            }
            std::swap(st.x, st.other);
            st.y = st.wb = nullptr;
        }
        if (L.mixer.kind == MixerSpec::PARALLEL) TRY(run_parallel(st, (int)r, w, L.mixer));
        else if (L.mixer.kind == MixerSpec::CHANNEL_DELTA) TRY(run_channel_delta(st, (int)r, w, L.mixer));
        else TRY(latent_attention(st, (int)r, w, L.mixer));
        st.y = n.y;
        st.wb = w.norm1b;
        if (L.mlp.kind == MlpSpec::NONE) continue;
        if (L.mlp.kind == MlpSpec::EXPERTS) {
            TRY(run_experts(st, w, L.mlp));
            st.y = n.y;
            st.wb = w.norm2b;
            continue;
        }
        TRY(linear(st, n.hmid, w.gu, DENSE_GEGLU, "linear_gateup_geglu", "gemv_norm_gateup_geglu", nullptr, w.norm2, PRO_RESIDUAL_NORM));
        TRY(linear(st, n.y, w.down, DENSE_T, "linear_down", "gemv_down", n.hmid, nullptr, PRO_ROWS));
        st.y = n.y;
        st.wb = w.norm2b;
    }

    // logits of the rows the caller asked for
    const int cnt = m.sel_count, V = s.vocab;
    AdvanceState adv{};  // a batch-1 decode model's step also moves the loop state on
    if (c.batch * c.seq_q == 1) adv = AdvanceState{m.d_ids, m.d_pos, m.d_past, m.d_active, m.d_tokens, m.d_step, m.token_cap};
    if (cnt) {
        ResidualNorm row = st.row(n.w->final_norm);
        row.x_out = nullptr;
        if (st.one) {
            int n_cand = 0;
            note(m, "gemv_norm_head", (double)V * n.ld * eb + st.row_bytes(eb) + V * 4.0, 2.0 * V * n.ld);
            TRY(dense_gemv(m.logits, nullptr, &row, PRO_RESIDUAL_NORM, n.w->head.w, V, n.ld, DENSE_F32, n.logit_scale, dt, m.stream, n.cand, &n_cand));
            note(m, adv.ids ? "greedy_advance" : "greedy_pick", n_cand * 8.0);
            TRY(greedy_pick(m.d_next, n.cand, n_cand, adv, m.stream));
        } else {
            note(m, "residual_norm", cnt * (st.row_bytes(eb) + n.ld * eb));
            TRY(residual_norm_rows(n.act, row, PRO_RESIDUAL_NORM, m.sel_first, m.sel_stride, cnt, dt, m.stream));
            note(m, "linear_head", (double)(V + cnt) * n.ld * eb + (double)cnt * V * 4, 2.0 * cnt * V * n.ld);
            TRY(dense_gemm(m.logits, n.act, n.w->head.w, cnt, V, n.ld, DENSE_F32, n.logit_scale, dt, m.stream));
        }
        // greedy token of every sequence whose last row is among them
        const float *lg = (const float *)m.logits;
        if (st.one) {
        } else if (S == 1 || (cnt == c.batch && (c.batch > 1 || m.sel_first == S - 1))) {
            note(m, adv.ids ? "argmax_advance" : "argmax_last", (double)c.batch * V * 4);
            TRY(argmax_rows<float>(m.d_next, lg, c.batch, V, adv, m.stream));
        } else if (c.batch > 1 || m.sel_first + cnt == S) {
            for (int b = 0; b < c.batch; b++) {
                const size_t last = c.batch > 1 ? (size_t)b * S + S - 1 : (size_t)cnt - 1;
                note(m, "argmax_last", (double)V * 4);
                TRY(argmax_rows<float>(m.d_next + b, lg + last * V, 1, V, AdvanceState{}, m.stream));
            }
        }
    }
    launch_timer() = LaunchTimer{};
    m.launches = (int)m.record.size();
    return 0;
}

// ---- a copy of the sequence states: what a run of the device loop computed past an end-of-sequence id is undone with it
bool model_has_sequence_state(const void *state) {
    const Model *m = (const Model *)state;
    return m && m->net && m->net->spec->sequence_state();
}
static int copy_state(Model &m, bool save) {
    LayeredNet &n = *m.net;
    size_t off = 0, total = 0;
    for (const StateSpec &st : n.spec->states) total += st.seq_floats * sizeof(float) * m.cfg.batch;
    if (save && !n.saved) MYNN_HIP(hipMalloc((void **)&n.saved, total));
    MYNN_REQUIRE(n.saved, MYNN_ERR_STATE, "sequence state: nothing saved");
    for (size_t r = 0; r < n.spec->runs.size(); r++) {
        if (!n.memory[r]) continue;
        const size_t bytes = n.spec->states[n.spec->runs[r].memory].seq_floats * sizeof(float) * m.cfg.batch;
        if (save) MYNN_HIP(hipMemcpyAsync(n.saved + off, n.memory[r], bytes, hipMemcpyDeviceToDevice, m.stream));
        else MYNN_HIP(hipMemcpyAsync(n.memory[r], n.saved + off, bytes, hipMemcpyDeviceToDevice, m.stream));
        off += bytes;
    }
    return 0;
}
int executor_save_state(void *state) { return copy_state(*(Model *)state, true); }
int executor_restore_state(void *state) { return copy_state(*(Model *)state, false); }

}  // namespace mynn
