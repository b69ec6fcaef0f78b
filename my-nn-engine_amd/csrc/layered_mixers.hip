// Mixers and feed-forwards of the layered executor beside latent attention: packing, scratch memory and launches of the
// parallel mixer (window attention and matrix memory), the gated delta rule and the experts.
//
// One new token: 4 launches for a parallel mixer (5 where the attention is cut into key ranges), 3 for a delta rule, 3 for the
// experts.  A parallel mixer's two halves share both projections: one matrix in front, one behind, whose input rows carry
// left_scale and right_scale.
#include <algorithm>
#include <cmath>

#include "layered.h"

namespace mynn {

int check_mixer(const MixerSpec &m) {
    if (m.kind == MixerSpec::PARALLEL)
        MYNN_REQUIRE(window_attention_dim_supported(pad_to(m.window.dim, 32)) && recurrent_dim_supported(pad_to(m.memory.dim, 4)), MYNN_ERR_UNSUPPORTED,
                     "attention heads of %d, memory heads of %d", m.window.dim, m.memory.dim);
    if (m.kind == MixerSpec::CHANNEL_DELTA)
        MYNN_REQUIRE(recurrent_dim_supported(pad_to(m.delta.dim, 4)), MYNN_ERR_UNSUPPORTED, "delta rule heads of %d", m.delta.dim);
    return 0;
}

// ---- weights ----------------------------------------------------------------------------------------------------------
int pack_parallel(WeightPacker &pk, LayerWeights &o, const MixerSpec &mix, const std::string &mx) {
    const ParallelDims d = parallel_dims(mix);
    const std::string l = mx + "left.", r = mx + "right.";
    TRY(pk.linear(o.in, d.n_in(), pk.ld));
    TRY(pk.rows(o.in, l + "q", d.H, d.dim, d.dimp, 0));
    TRY(pk.rows(o.in, l + "k", d.G, d.dim, d.dimp, d.qcols()));
    TRY(pk.rows(o.in, r + "q", d.R, d.rd, d.rdp, d.mem_q()));
    TRY(pk.rows(o.in, r + "k", d.R, d.rd, d.rdp, d.mem_k()));
    TRY(pk.rows(o.in, r + "v", d.R, d.rv, d.rvp, d.mem_v()));
    TRY(pk.rows(o.in, r + "g", d.R, d.rv, d.rvp, d.mem_g()));
    TRY(pk.rows(o.in, r + "i", 1, d.R, d.R, d.mem_i()));
    TRY(pk.rows(o.in, r + "f", 1, d.R, d.R, d.mem_f()));
    TRY(pk.alloc((void **)&o.taps, d.taps, d.conv(), sizeof(float)));
    TRY(pack_taps(PackTaps{o.taps, pk.src(l + "q.conv"), d.conv(), 0, d.H, d.dim, d.dimp, d.taps}, pk.dt, pk.m.stream));
    TRY(pack_taps(PackTaps{o.taps, pk.src(l + "k.conv"), d.conv(), d.qcols(), d.G, d.dim, d.dimp, d.taps}, pk.dt, pk.m.stream));
    TRY(pk.vec(&o.q_norm, l + "q.norm", d.H, d.dim, d.dimp, d.H * d.dimp));
    TRY(pk.vec(&o.k_norm, l + "k.norm", d.G, d.dim, d.dimp, d.G * d.dimp));
    TRY(pk.vec(&o.head_norm, r + "norm", d.R, d.rv, d.rvp, d.R * d.rvp));
    TRY(pk.norm(&o.i_bias, r + "i.b", d.R, d.R));
    TRY(pk.norm(&o.f_bias, r + "f.b", d.R, d.R));
    TRY(pk.linear(o.o, pk.ld, d.acols()));
    TRY(pk.cols(o.o, l + "o", d.H, d.dim, d.dimp, 0));
    return pk.cols(o.o, r + "o", d.R, d.rv, d.rvp, d.qcols());
}

int pack_channel_delta(WeightPacker &pk, LayerWeights &o, const MixerSpec &mix, const std::string &mx) {
    const DeltaDims d = delta_dims(mix.delta);
    TRY(pk.linear(o.in, d.n_in(), pk.ld));
    TRY(pk.rows(o.in, mx + "q", d.G, d.d, d.dp, 0));
    TRY(pk.rows(o.in, mx + "k", d.G, d.d, d.dp, d.col_k()));
    TRY(pk.rows(o.in, mx + "v", d.H, d.v, d.vp, d.col_v()));
    TRY(pk.rows(o.in, mx + "b", 1, d.H, d.H, d.col_b()));
    TRY(pk.rows(o.in, mx + "a1", 1, d.ra, d.ra, d.col_low()));
    TRY(pk.rows(o.in, mx + "g1", 1, d.rg, d.rg, d.col_low() + d.rap));
    TRY(pk.alloc((void **)&o.taps, d.taps, d.conv(), sizeof(float)));
    TRY(pack_taps(PackTaps{o.taps, pk.src(mx + "q.conv"), d.conv(), 0, d.G, d.d, d.dp, d.taps}, pk.dt, pk.m.stream));
    TRY(pack_taps(PackTaps{o.taps, pk.src(mx + "k.conv"), d.conv(), d.col_k(), d.G, d.d, d.dp, d.taps}, pk.dt, pk.m.stream));
    TRY(pack_taps(PackTaps{o.taps, pk.src(mx + "v.conv"), d.conv(), d.col_v(), d.H, d.v, d.vp, d.taps}, pk.dt, pk.m.stream));
    // both second maps over the two low-rank parts side by side, zeros where a row does not look
    TRY(pk.linear(o.low, d.n_low(), d.low()));
    TRY(pack_blocks(PackBlocks{o.low.w, pk.src(mx + "a2"), d.low(), d.ra, d.H, d.d, 0, d.dp, 0, d.d, 1, d.ra, 0, d.ra, d.ra, 0, 0}, pk.dt, pk.m.stream));
    TRY(pack_blocks(PackBlocks{o.low.w, pk.src(mx + "g2"), d.low(), d.rg, d.H, d.v, d.H * d.dp, d.vp, 0, d.v, 1, d.rg, d.rap, d.rg, d.rg, 0, 0}, pk.dt, pk.m.stream));
    TRY(pk.norm(&o.a_log, mx + "A_log", d.H, d.H));
    TRY(pk.vec(&o.dt_bias, mx + "dt_bias", d.H, d.d, d.dp, d.H * d.dp));
    TRY(pk.norm(&o.head_norm, mx + "norm", d.v, d.vp));
    TRY(pk.linear(o.o, pk.ld, d.acols()));
    return pk.cols(o.o, mx + "o", d.H, d.v, d.vp, 0);
}

int pack_experts(WeightPacker &pk, LayerWeights &o, const MlpSpec &mlp, const std::string &p) {
    const int W = pk.s.width, F = mlp.ff, Fp = pad_to(F, 64);
    TRY(pk.linear(o.router, mlp.experts, pk.ld));
    TRY(pk.rows(o.router, p + "router", 1, mlp.experts, mlp.experts, 0));
    TRY(pk.alloc(&o.gu.w, (size_t)mlp.experts * 2 * Fp, pk.ld));
    TRY(pk.alloc(&o.down.w, (size_t)mlp.experts * pk.ld, Fp));
    o.gu.N = 2 * Fp;
    o.gu.K = o.down.N = pk.ld;
    o.down.K = Fp;
    const size_t eb = dtype_size(pk.dt);
    for (int e = 0; e < mlp.experts; e++) {
        const std::string x = p + "e" + std::to_string(e) + ".";
        void *gu = (char *)o.gu.w + (size_t)e * 2 * Fp * pk.ld * eb, *down = (char *)o.down.w + (size_t)e * pk.ld * Fp * eb;
        TRY(pack_blocks(PackBlocks{gu, pk.src(x + "gate"), pk.ld, W, 1, F, 0, F, 0, F, 1, W, 0, W, W, 32, 0}, pk.dt, pk.m.stream));
        TRY(pack_blocks(PackBlocks{gu, pk.src(x + "up"), pk.ld, W, 1, F, 0, F, 0, F, 1, W, 0, W, W, 32, 1}, pk.dt, pk.m.stream));
        TRY(pack_blocks(PackBlocks{down, pk.src(x + "down"), Fp, F, 1, W, 0, W, 0, W, 1, F, 0, F, F, 0, 0}, pk.dt, pk.m.stream));
    }
    return 0;
}

// ---- scratch memory -------------------------------------------------------------------------------------------------------
static void grow(size_t &v, size_t n) { v = std::max(v, n); }

void scratch_recurrent(MixerScratch &x, const MixerSpec &mix, const mynn_model_config &c) {
    const size_t rows = (size_t)c.batch * c.seq_q, eb = dtype_size(c.dtype);
    const bool many = c.seq_q > 1;
    if (mix.kind == MixerSpec::PARALLEL) {
        const ParallelDims d = parallel_dims(mix);
        grow(x.proj, rows * d.n_in() * 4);
        grow(x.q, rows * d.qcols() * eb);
        for (int S = 1; S <= c.seq_q; S++) {
            const size_t ns = window_attention_splits(c.batch, S, d, mix.window.window, mix.window.keep_first, c.max_seq);
            if (ns == 1) break;  // (nor for any more rows)
            grow(x.part_o, (size_t)c.batch * S * d.H * ns * d.dimp * 4);
            grow(x.part_ml, (size_t)c.batch * S * d.H * ns * 2 * 4);
        }
        if (many) {
            grow(x.gates, rows * d.R * 16);
            grow(x.o, rows * d.R * pad_to(d.rv + 1, 4) * 4);
            grow(x.blocks, recurrent_block_floats(c.batch, c.seq_q, d.R, d.rdp, false) * 4);
        }
    } else if (mix.kind == MixerSpec::CHANNEL_DELTA) {
        const DeltaDims d = delta_dims(mix.delta);
        grow(x.proj, rows * d.n_in() * 4);
        if (!many) return;
        grow(x.qk, rows * 2 * d.G * d.dp * 4);
        grow(x.v, rows * d.H * d.vp * 4);
        grow(x.beta, rows * d.H * 4);
        grow(x.blocks, recurrent_block_floats(c.batch, c.seq_q, d.H, d.dp, true) * 4);
        grow(x.low, rows * d.low() * eb);
        grow(x.dec, rows * d.n_low() * 4);
        grow(x.o, rows * d.H * d.vp * 4);
    }
}

void scratch_experts(MixerScratch &x, const MlpSpec &mlp, const mynn_model_config &c, int ld) {
    const size_t eb = dtype_size(c.dtype), fp = pad_to(mlp.ff, 64), rows = (size_t)c.batch * c.seq_q, a = rows * mlp.top;
    grow(x.router, (size_t)mlp.experts * 4);
    grow(x.hmid, mlp.top * fp * eb);
    grow(x.chosen, (size_t)mlp.top * 4);
    // (shorter portions may take the smaller tiles: more of them, fewer rows)
    const int gr = expert_group_rows((int)rows, mlp.experts, mlp.top);
    const size_t tiles = expert_tiles((int)rows, mlp.experts, mlp.top, 128), slots = (size_t)gr * expert_tiles((int)rows, mlp.experts, mlp.top, gr);
    grow(x.choice, a * 4);
    grow(x.score, a * 4);
    grow(x.tile_group, tiles * 4);
    grow(x.slot, slots * 4);
    grow(x.hsort, slots * fp * eb);
    if (mlp.top > 1) grow(x.parts, a * ld * 4);
}

// ---- launches -------------------------------------------------------------------------------------------------------------
int run_parallel(Stream &st, int run, const LayerWeights &w, const MixerSpec &mix) {
    Model &m = st.m;
    LayeredNet &n = st.n;
    const mynn_model_config &c = m.cfg;
    const ParallelDims d = parallel_dims(mix);
    const double eb = dtype_size(c.dtype), rows = st.rows;
    const int S = m.rows_now, B = c.batch;
    TRY(linear(st, n.proj, w.in, DENSE_F32, "linear_parallel_in", "gemv_parallel_in", nullptr, nullptr, PRO_RESIDUAL));
    WindowAttnParams a{};
    a.d = d; a.window = mix.window.window; a.keep_first = mix.window.keep_first; a.scale = mix.window.scale; a.out_scale = mix.left_scale; a.eps = n.spec->eps;
    a.rot_dims = mix.window.rot.dims; a.rot = n.rot[n.spec->runs[run].layer]; a.proj = (const float *)n.proj; a.conv_w = w.taps;
    a.q_norm = w.q_norm; a.k_norm = w.k_norm; a.ring = n.memory[run] + d.st_ring(); a.state_stride = d.state(); a.q = n.q; a.cache = n.caches[run];
    a.paging = m.paging; a.d_past = m.d_past; a.B = B; a.S = S; a.max_seq = c.max_seq; a.out = n.attn; a.part_o = n.part_o; a.part_ml = n.part_ml;
    MemoryParams r{};
    r.d = d; r.cap = mix.memory.gate_cap; r.out_scale = mix.right_scale; r.eps = n.spec->eps; r.q_scale = 1.0f / sqrtf((float)d.rd);
    r.proj = (const float *)n.proj; r.i_bias = w.i_bias; r.f_bias = w.f_bias; r.norm = w.head_norm; r.state = n.memory[run]; r.state_stride = d.state();
    r.d_past = m.d_past; r.B = B; r.S = S; r.out = n.attn; r.gates = n.gates; r.o = n.o; r.blocks = n.blocks;
    const double prep = rows * (d.conv() * 4.0 + (d.qcols() + d.row()) * eb), mem = 2.0 * B * d.st_max() * 4.0, memio = rows * d.R * (2.0 * d.rdp + d.rvp) * 4;
    note(m, S == 1 ? "attention_prepare_memory_step" : "attention_prepare", S == 1 ? prep + mem + memio + rows * d.R * d.rvp * (4 + eb) : prep + rows * d.R * 24.0);
    TRY(parallel_prepare(a, r, c.dtype, m.stream));
    const bool tiles = S > 1 && window_prefill_supported(d, c.dtype);
    a.nsplit = tiles ? 1 : window_attention_splits(B, S, d, a.window, a.keep_first, c.max_seq);
    if (tiles) {
        // keys a row sees: its window and the kept tokens
        const double past = m.h_past, win = a.window ? a.window : past + S, sees = std::min<double>(past + 0.5 * S, win + a.keep_first);
        note(m, "window_attention", rows * (2.0 * d.qcols()) * eb + B * std::min(past + S, S + win + a.keep_first) * d.row() * eb, 4.0 * d.H * d.dim * rows * sees);
        TRY(window_attention_prefill(a, m.h_past, c.dtype, m.stream));
    } else {
        // (bytes: queries only; the cache rows read depend on the context, which the host does not know under replay)
        note(m, "window_attention", rows * d.qcols() * eb);
        TRY(window_attention_rows(a, c.dtype, m.stream));
        if (a.nsplit > 1) {
            note(m, "window_merge", rows * d.H * (d.dimp * (4.0 * a.nsplit + eb)));
            TRY(window_attention_merge(a, c.dtype, m.stream));
        }
    }
    if (S > 1) {
        const double ops = recurrent_block_floats(B, S, d.R, d.rdp, false) * 4.0;
        note(m, "memory_blocks", rows * d.R * 2.0 * d.rdp * 4 + ops);
        TRY(memory_blocks(r, m.stream));
        note(m, "memory_recurrence", ops + mem + rows * d.R * (d.rvp + d.rv + 1.0) * 4, 4.0 * rows * d.R * (d.rd + 8) * (d.rv + 1));
        TRY(memory_recurrence(r, m.stream));
        note(m, "head_norm_gate", rows * d.R * d.rvp * (8.0 + eb));
        TRY(memory_out(a, r, c.dtype, m.stream));
    }
    return linear(st, n.y, w.o, DENSE_T, "linear_o", "gemv_o", n.attn, nullptr, PRO_ROWS);
}

int run_channel_delta(Stream &st, int run, const LayerWeights &w, const MixerSpec &mix) {
    Model &m = st.m;
    LayeredNet &n = st.n;
    const mynn_model_config &c = m.cfg;
    const DeltaDims d = delta_dims(mix.delta);
    const double eb = dtype_size(c.dtype), rows = st.rows;
    const int S = m.rows_now, B = c.batch;
    TRY(linear(st, n.proj, w.in, DENSE_F32, "linear_delta_in", "gemv_delta_in", nullptr, nullptr, PRO_RESIDUAL));
    DeltaParams p{};
    p.d = d; p.eps = n.spec->eps; p.proj = (const float *)n.proj; p.conv_w = w.taps; p.low_w = w.low.w; p.a_log = w.a_log; p.dt_bias = w.dt_bias;
    p.norm = w.head_norm; p.state = n.memory[run]; p.state_stride = d.state(); p.d_past = m.d_past; p.B = B; p.S = S; p.out = n.attn;
    p.qk = n.qk; p.v = n.v; p.beta = n.beta; p.blocks = n.blocks; p.low = n.low; p.dec = n.dec; p.o = n.o;
    const double state = 2.0 * B * d.H * d.v * d.dp * 4.0;
    if (S == 1) {
        note(m, "delta_step", state + (double)w.low.N * w.low.K * eb / 2 + rows * (d.n_in() * 4.0 + d.acols() * eb + 2.0 * d.taps * d.conv() * 4));
        TRY(delta_step(p, c.dtype, m.stream));
    } else {
        note(m, "delta_prepare", rows * (d.n_in() * 4.0 + d.conv() * 4.0 + d.low() * eb));
        TRY(delta_prepare(p, c.dtype, m.stream));
        note(m, "linear_delta_low", ((double)w.low.N * w.low.K + rows * w.low.K) * eb + rows * w.low.N * 4, 2.0 * rows * w.low.N * w.low.K);
        TRY(dense_gemm(n.dec, n.low, w.low.w, st.rows, w.low.N, w.low.K, DENSE_F32, nullptr, c.dtype, m.stream));
        const double ops = recurrent_block_floats(B, S, d.H, d.dp, true) * 4.0;
        note(m, "delta_blocks", rows * (2.0 * d.G * d.dp + d.H * d.dp) * 4 + ops);
        TRY(delta_blocks(p, c.dtype, m.stream));
        note(m, "delta_recurrence", state + ops + rows * d.H * 2.0 * d.vp * 4, 6.0 * rows * d.H * (d.d + 11) * d.v);
        TRY(delta_recurrence(p, m.stream));
        note(m, "head_norm_gate", rows * d.H * d.vp * (8.0 + eb));
        TRY(delta_out(p, c.dtype, m.stream));
    }
    return linear(st, n.y, w.o, DENSE_T, "linear_o", "gemv_o", n.attn, nullptr, PRO_ROWS);
}

int run_experts(Stream &st, const LayerWeights &w, const MlpSpec &mlp) {
    Model &m = st.m;
    LayeredNet &n = st.n;
    const int dt = m.cfg.dtype, fp = w.down.K, ld = n.ld;
    const double eb = dtype_size(dt), rows = st.rows, gu = (double)w.gu.N * w.gu.K, down = (double)w.down.N * w.down.K;
    ExpertParams p{};
    p.E = mlp.experts; p.top = mlp.top; p.ld = ld; p.fp = fp; p.gu = w.gu.w; p.down = w.down.w; p.y = n.y; p.rows = st.rows;
    if (st.one) {
        TRY(linear(st, n.router, w.router, DENSE_F32, "linear_router", "gemv_router", nullptr, nullptr, PRO_RESIDUAL));
        p.x = st.x; p.logits = n.router; p.hmid = n.hmid; p.chosen = n.chosen;
        note(m, "gemv_experts_gateup", mlp.top * (gu + fp) * eb + ld * 4.0, 2.0 * mlp.top * gu);
        TRY(expert_gateup_row(p, dt, m.stream));
        note(m, "gemv_experts_down", mlp.top * (down + fp) * eb + ld * eb, 2.0 * mlp.top * down);
        return expert_down_row(p, dt, m.stream);
    }
    note(m, "residual_norm", rows * (st.row_bytes(eb) + ld * eb));
    TRY(residual_norm_rows(n.act, st.row(nullptr), PRO_RESIDUAL, 0, 1, st.rows, dt, m.stream));
    st.added();
    p.x = st.x; p.router = w.router.w; p.act = n.act; p.choice = n.choice; p.score = n.score; p.tile_expert = n.tile_group; p.slot = n.slot;
    p.hsort = n.hsort; p.parts = n.parts;
    const double a = rows * mlp.top, used = std::min<double>(mlp.experts, a);
    note(m, "expert_route", rows * ld * 4.0 + (double)mlp.experts * ld * eb, 2.0 * rows * mlp.experts * ld);
    TRY(expert_route(p, dt, m.stream));
    note(m, "expert_sort", a * 12.0);
    TRY(expert_sort(p, m.stream));
    note(m, "linear_experts_gateup", (used * gu + rows * ld + a * fp) * eb, 2.0 * a * gu);
    TRY(expert_gateup(p, dt, m.stream));
    note(m, "linear_experts_down", (used * down + a * fp) * eb + a * ld * (mlp.top > 1 ? 4.0 : eb), 2.0 * a * down);
    TRY(expert_down(p, dt, m.stream));
    if (mlp.top > 1) {
        note(m, "expert_sum", a * ld * 4.0 + rows * ld * eb);
        TRY(expert_sum(p, dt, m.stream));
    }
    return 0;
}

}  // namespace mynn
