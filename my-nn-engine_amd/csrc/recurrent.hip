// Recurrent mixers (see recurrent.h).  A state column -- one value channel of a head -- is a recurrence of its own given the
// keys, queries and gates, so a head's columns are spread over lanes and workgroups.
//
// One new token: delta_step_kernel / the memory workgroups of parallel_prepare_kernel, one workgroup per head, do everything
// between the two projections; the first state columns are requested before anything else.
// Several tokens: the elementwise parts run over all rows at once, then the tokens go through the recurrence sixteen at a time.
// With S the state in front of a block, G_j the product of its decays up to token j, and u_i what token i writes,
//     u_j = beta_j (v_j - (G_j k_j) . S - sum_{i<j} A_ji u_i),  A_ji = k_j . (g_{i+1} .. g_j k_i)
//     o_j = (G_j q_j) . S + sum_{i<=j} B_ji u_i,                B_ji = q_j . (g_{i+1} .. g_j k_i)
//     S  <- G_16 S + sum_i (g_{i+1} .. g_16 k_i) u_i
// (products of decays only, no quotients).  What does not depend on the values -- G k, G q, the keys carried to the block's
// end, B and the inverse T of the triangular system -- is made for all blocks in parallel (delta_blocks_kernel,
// memory_blocks_kernel, whose u_i is the value itself); recurrence_kernel then walks the blocks with f32 matrix-core products.
#include <algorithm>
#include <type_traits>

#include "dense_load.h"
#include "recurrent.h"

namespace mynn {

__device__ inline float softplusf(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ inline float4 silu4(const float4 &x) { return float4{x.x * sigmoidf(x.x), x.y * sigmoidf(x.y), x.z * sigmoidf(x.z), x.w * sigmoidf(x.w)}; }

// f(LC, RP): lanes per column and key channels per lane
template <typename F> static int dispatch_columns(int dp, F &&f) {
    using std::integral_constant;
    if (dp <= 32) return f(integral_constant<int, 8>{}, integral_constant<int, 4>{});
    if (dp <= 64) return f(integral_constant<int, 16>{}, integral_constant<int, 4>{});
    if (dp <= 128) return f(integral_constant<int, 32>{}, integral_constant<int, 4>{});
    if (dp <= 256) return f(integral_constant<int, 32>{}, integral_constant<int, 8>{});
    return f(integral_constant<int, 32>{}, integral_constant<int, 16>{});
}
bool recurrent_dim_supported(int dp) { return dp <= 512; }

// ---- a state column of one lane group: key channels P * 4 LC + 4 r .. + 3, P < RP / 4, of lane r ----------------------
template <int LC, int RP> struct Column {
    float s[RP];
    __device__ static int channel(int r, int P) { return P * 4 * LC + 4 * r; }
    __device__ void load(const float *at, int r, int dp) {
#pragma unroll
        for (int P = 0; P < RP / 4; P++) *(float4 *)(s + 4 * P) = *(const float4 *)(at + min(channel(r, P), dp - 4));
    }
    __device__ void clear(bool all, int r, int dp) {
#pragma unroll
        for (int P = 0; P < RP / 4; P++)
            if (all || channel(r, P) >= dp) s[4 * P] = s[4 * P + 1] = s[4 * P + 2] = s[4 * P + 3] = 0.f;
    }
    __device__ void store(float *at, int r, int dp) const {
#pragma unroll
        for (int P = 0; P < RP / 4; P++)
            if (channel(r, P) < dp) *(float4 *)(at + channel(r, P)) = *(const float4 *)(s + 4 * P);
    }
};
// a vector over key channels in LDS, [4 LC * RP / 4] values
template <int LC, int RP> __device__ inline void channels_of(const float *vec, int r, float *f) {
#pragma unroll
    for (int P = 0; P < RP / 4; P++) *(float4 *)(f + 4 * P) = *(const float4 *)(vec + Column<LC, RP>::channel(r, P));
}

// ---- one new token ------------------------------------------------------------------------------------------------------
constexpr int kStepThreads = 512, kStepWaves = kStepThreads / 64;

// sum over the workgroup; every thread gets it
template <int NT> __device__ inline float block_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; w++) t += red[w];
    return t;
}

template <typename T, int LC, int RP>
__global__ __launch_bounds__(kStepThreads) void delta_step_kernel(DeltaParams p) {
    constexpr int KD = LC * RP, CPP = kStepWaves * 64 / LC, PRE = 32 / RP;  // columns per pass, passes requested together
    extern __shared__ __align__(16) float sm[];
    __shared__ float red[kStepWaves], qk_sums[2];
    const DeltaDims &d = p.d;
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int r = lane % LC, cg = wave * (64 / LC) + lane / LC, hk = h / (d.H / d.G);
    float *qs = sm, *ks = qs + KD, *gs = ks + KD, *vs = gs + KD, *os = vs + d.vp, *gate = os + d.vp, *low = gate + d.vp;
    const float *proj = p.proj + (size_t)b * d.n_in();
    float *state = p.state + (size_t)b * p.state_stride, *ring = state + d.st_ring(), *cols = state + (size_t)h * d.v * d.dp;
    const int past = *p.d_past, passes = (d.v + CPP - 1) / CPP;
    Column<LC, RP> st[PRE];
    auto request = [&](int pass0) {
#pragma unroll
        for (int i = 0; i < PRE; i++) st[i].load(cols + (size_t)min((pass0 + i) * CPP + cg, d.v - 1) * d.dp, r, d.dp);
    };
    request(0);

    for (int i = tid; i < KD; i += kStepThreads) gs[i] = 0.f;
    for (int i = tid; i < d.low(); i += kStepThreads) low[i] = proj[d.col_low() + i];
    const bool keeps = h % (d.H / d.G) == 0;  // (the heads of a group share q and k; one of them stores the ring)
    for (int i = tid * 4; i < 2 * KD + d.vp; i += kStepThreads * 4) {
        int ch = -1;
        if (i < KD) ch = i < d.dp ? hk * d.dp + i : -1;
        else if (i < 2 * KD) ch = i - KD < d.dp ? d.col_k() + hk * d.dp + i - KD : -1;
        else ch = d.col_v() + h * d.vp + i - 2 * KD;
        float4 y = float4{0.f, 0.f, 0.f, 0.f};
        if (ch >= 0) {
            y = silu4(short_conv4(p.conv_w, proj, 0, ring, ch, d.conv(), d.taps, 0, past));
            if (keeps || i >= 2 * KD) *(float4 *)(ring + (size_t)(past % d.taps) * d.conv() + ch) = *(const float4 *)(proj + ch);
        }
        *(float4 *)(i < 2 * KD ? qs + i : vs + i - 2 * KD) = y;  // (ks follows qs)
    }
    __syncthreads();
    if (wave < 2) {
        const float *x = wave ? ks : qs;
        float ss = 0.f;
        for (int i = lane; i < KD; i += 64) ss = fmaf(x[i], x[i], ss);
        ss = wave_sum(ss);
        if (lane == 0) qk_sums[wave] = (wave ? 1.f : 1.0f / sqrtf((float)d.d)) / sqrtf(ss + 1e-6f);
    }
    // decays and gates: eight lanes per row of the second map
    {
        const T *lw = (const T *)p.low_w;
        const int sub = tid & 7;
        const float ea = expf(Elem<T>::ld((const T *)p.a_log, h));
        for (int i = tid >> 3; i < d.dp + d.vp; i += kStepThreads / 8) {  // (all lanes of a group of eight together)
            const bool dec = i < d.dp;
            const int row = dec ? h * d.dp + i : d.H * d.dp + h * d.vp + i - d.dp;
            const T *w = lw + (size_t)row * d.low() + (dec ? 0 : d.rap);
            const float *x = low + (dec ? 0 : d.rap);
            float a = 0.f;
            for (int c = sub * 8; c < (dec ? d.rap : d.rgp); c += 64) {
                float f[8];
                load8<T>(w + c, f);
#pragma unroll
                for (int e = 0; e < 8; e++) a = fmaf(f[e], x[c + e], a);
            }
            a = group_sum<8>(a);
            if (sub == 0) {
                if (dec) gs[i] = expf(-ea * softplusf(a + Elem<T>::ld((const T *)p.dt_bias, h * d.dp + i)));
                else gate[i - d.dp] = sigmoidf(a);
            }
        }
    }
    __syncthreads();
    float q[RP], k[RP], g[RP];
    channels_of<LC, RP>(qs, r, q);
    channels_of<LC, RP>(ks, r, k);
    channels_of<LC, RP>(gs, r, g);
    const float qn = qk_sums[0], kn = qk_sums[1], beta = sigmoidf(proj[d.col_b() + h]);
#pragma unroll
    for (int i = 0; i < RP; i++) {
        q[i] *= qn;
        k[i] *= kn;
    }
    float ss = 0.f;
    for (int pass0 = 0; pass0 < passes; pass0 += PRE) {
        if (pass0) request(pass0);
#pragma unroll
        for (int i = 0; i < PRE; i++) {
            const int col = (pass0 + i) * CPP + cg;
            Column<LC, RP> &S = st[i];
            S.clear(past == 0, r, d.dp);
            float a = 0.f, o = 0.f;
#pragma unroll
            for (int j = 0; j < RP; j++) {
                S.s[j] *= g[j];
                a = fmaf(S.s[j], k[j], a);
            }
            a = group_sum<LC>(a);
            const float u = beta * (vs[min(col, d.v - 1)] - a);
#pragma unroll
            for (int j = 0; j < RP; j++) {
                S.s[j] = fmaf(k[j], u, S.s[j]);
                o = fmaf(S.s[j], q[j], o);
            }
            o = group_sum<LC>(o);
            if (col < d.v) {
                S.store(cols + (size_t)col * d.dp, r, d.dp);
                if (r == 0) {
                    os[col] = o;
                    ss = fmaf(o, o, ss);
                }
            }
        }
    }
    const float inv = 1.0f / sqrtf(block_sum<kStepThreads>(ss, red) / (float)d.v + p.eps);
    T *out = (T *)p.out + (size_t)b * d.acols() + h * d.vp;
    for (int c = tid; c < d.vp; c += kStepThreads)
        Elem<T>::st(out, c, c < d.v ? os[c] * inv * Elem<T>::ld((const T *)p.norm, c) * gate[c] : 0.f);
}

struct MemoryGates {
    float in, forget;
};
__device__ inline MemoryGates memory_gates(float cap, float zi, float zf) {
    return MemoryGates{cap * tanhf(zi / cap), -softplusf(-cap * tanhf(zf / cap))};
}

template <typename T, int LC, int RP>
__device__ inline void memory_step(const MemoryParams &p, int head, int b, float *sm, float *red) {
    constexpr int KD = LC * RP, CPP = kStepWaves * 64 / LC, PRE = 32 / RP;
    const ParallelDims &d = p.d;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane % LC, cg = wave * (64 / LC) + lane / LC;
    float *qs = sm, *ks = qs + KD, *os = ks + KD;
    const float *proj = p.proj + (size_t)b * d.n_in();
    float *state = p.state + (size_t)b * p.state_stride, *cols = state + (size_t)head * (d.rv + 1) * d.rdp, *mx = state + d.st_max() + head;
    const int past = *p.d_past, ncol = d.rv + 1, passes = (ncol + CPP - 1) / CPP;
    Column<LC, RP> st[PRE];
    auto request = [&](int pass0) {
#pragma unroll
        for (int i = 0; i < PRE; i++) st[i].load(cols + (size_t)min((pass0 + i) * CPP + cg, ncol - 1) * d.rdp, r, d.rdp);
    };
    request(0);
    const float m_old = past ? *mx : 0.f;
    const MemoryGates gt = memory_gates(p.cap, proj[d.mem_i() + head] + Elem<T>::ld((const T *)p.i_bias, head), proj[d.mem_f() + head] + Elem<T>::ld((const T *)p.f_bias, head));
    const float m_new = fmaxf(gt.forget + m_old, gt.in), keep = expf(gt.forget + m_old - m_new), put = expf(gt.in - m_new);
    for (int i = tid; i < 2 * KD; i += kStepThreads) {
        const int c = i < KD ? i : i - KD;
        float x = 0.f;
        if (c < d.rdp) x = i < KD ? proj[d.mem_q() + head * d.rdp + c] * p.q_scale : proj[d.mem_k() + head * d.rdp + c];
        qs[i] = x;
    }
    __syncthreads();
    float q[RP], k[RP];
    channels_of<LC, RP>(qs, r, q);
    channels_of<LC, RP>(ks, r, k);
    for (int pass0 = 0; pass0 < passes; pass0 += PRE) {
        if (pass0) request(pass0);
#pragma unroll
        for (int i = 0; i < PRE; i++) {
            const int col = (pass0 + i) * CPP + cg;
            Column<LC, RP> &S = st[i];
            S.clear(past == 0, r, d.rdp);
            const float v = put * (col < d.rv ? proj[d.mem_v() + head * d.rvp + col] : 1.f);
            float o = 0.f;
#pragma unroll
            for (int j = 0; j < RP; j++) {
                S.s[j] = fmaf(k[j], v, keep * S.s[j]);
                o = fmaf(S.s[j], q[j], o);
            }
            o = group_sum<LC>(o);
            if (col < ncol) {
                S.store(cols + (size_t)col * d.rdp, r, d.rdp);
                if (r == 0) os[col] = o;
            }
        }
    }
    __syncthreads();  // (also: every thread has read the old maximum)
    if (tid == 0) *mx = m_new;
    const float den = 1.0f / (fmaxf(fabsf(os[d.rv]), expf(-m_new)) + 1e-6f);
    float ss = 0.f;
    for (int c = tid; c < d.rv; c += kStepThreads) {
        const float o = os[c] * den;
        ss = fmaf(o, o, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum<kStepThreads>(ss, red) / (float)d.rv + p.eps) * den;
    T *out = (T *)p.out + (size_t)b * d.acols() + d.qcols() + head * d.rvp;
    for (int c = tid; c < d.rvp; c += kStepThreads)
        Elem<T>::st(out, c, c < d.rv ? os[c] * inv * Elem<T>::ld((const T *)p.norm, head * d.rvp + c) *
                                           sigmoidf(proj[d.mem_g() + head * d.rvp + c]) * p.out_scale : 0.f);
}

// Gates of all tokens of a portion, one wave per (sequence, head).  The running maximum is a scan over maps
// m -> max(f + m, i), 64 tokens at a time.  (A maximum that is off by a rounding scales state, normaliser and floor alike.)
template <typename T> __device__ inline void memory_gate_scan(const MemoryParams &p, int head, int b) {
    const ParallelDims &d = p.d;
    const int lane = threadIdx.x & 63;
    float *mx = p.state + (size_t)b * p.state_stride + d.st_max() + head;
    float m = *p.d_past ? *mx : 0.f;
    auto row_at = [&](int t0) { return (size_t)b * p.S + min(t0 + lane, p.S - 1); };
    auto raw = [&](int t0) {
        const float *proj = p.proj + row_at(t0) * d.n_in();
        return float2{proj[d.mem_i() + head], proj[d.mem_f() + head]};
    };
    const float ib = Elem<T>::ld((const T *)p.i_bias, head), fb = Elem<T>::ld((const T *)p.f_bias, head);
    float2 next = raw(0);
    for (int t0 = 0; t0 < p.S; t0 += 64) {
        const int n = min(64, p.S - t0);
        const size_t row = row_at(t0);
        const MemoryGates gt = memory_gates(p.cap, next.x + ib, next.y + fb);
        next = raw(t0 + 64);
        float f = gt.forget, i = gt.in;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float fo = __shfl_up(f, off, 64), io = __shfl_up(i, off, 64);
            if (lane >= off) {
                i = fmaxf(f + io, i);
                f += fo;
            }
        }
        const float after = fmaxf(f + m, i), shifted = __shfl_up(after, 1, 64), before = lane ? shifted : m;
        if (lane < n) *(float4 *)(p.gates + (row * d.R + head) * 4) = float4{expf(gt.forget + before - after), expf(gt.in - after), expf(-after), 0.f};
        m = __shfl(after, n - 1, 64);
    }
    if (lane == 0) *mx = m;
}

// one workgroup per (sequence, memory head), then two per row: queries and keys of the attention
template <typename T, bool STEP, int LC, int RP>
__global__ __launch_bounds__(STEP ? kStepThreads : 256) void parallel_prepare_kernel(WindowAttnParams a, MemoryParams m) {
    constexpr int NT = STEP ? kStepThreads : 256;
    extern __shared__ __align__(16) float sm[];
    __shared__ float red[NT / 64];
    const int heads = a.B * a.d.R, id = blockIdx.x;
    if (id >= heads) {
        window_prepare_row<T, NT>(a, (id - heads) >> 1, (id - heads) & 1, sm, red);
        return;
    }
    const int head = id % a.d.R, b = id / a.d.R;
    if constexpr (STEP) memory_step<T, LC, RP>(m, head, b, sm, red);
    else if (threadIdx.x < 64) memory_gate_scan<T>(m, head, b);
}

constexpr size_t kLdsMax = 152 * 1024;
template <typename K> static int raise_lds(K kernel, size_t lds) {
    MYNN_REQUIRE(lds <= kLdsMax, MYNN_ERR_UNSUPPORTED, "recurrent mixer: %zu bytes of LDS", lds);
    if (lds > 60 * 1024) MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsMax));
    return 0;
}

static int check_delta(const DeltaParams &p) {
    MYNN_REQUIRE(p.proj && p.conv_w && p.state && p.d_past && p.B > 0 && p.S > 0 && recurrent_dim_supported(p.d.dp), MYNN_ERR_INVALID, "delta rule: bad operand");
    return 0;
}

int delta_step(const DeltaParams &p, int dtype, hipStream_t s) {
    int rc = check_delta(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.S == 1 && p.out && p.low_w && p.a_log && p.dt_bias && p.norm && p.B <= 65535, MYNN_ERR_INVALID, "delta step: bad operand");
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        return dispatch_columns(p.d.dp, [&](auto lc, auto rp) {
            constexpr int LC = decltype(lc)::value, RP = decltype(rp)::value;
            auto kernel = delta_step_kernel<T, LC, RP>;
            const size_t lds = (size_t)(3 * LC * RP + 3 * p.d.vp + p.d.low()) * 4;
            int rc2 = raise_lds(kernel, lds);
            if (rc2) return rc2;
            MYNN_LAUNCH(kernel, dim3(p.d.H, p.B), dim3(kStepThreads), lds, s, p);
            return launch_status("delta_step_kernel");
        });
    });
}

int parallel_prepare(const WindowAttnParams &a, const MemoryParams &m, int dtype, hipStream_t s) {
    MYNN_REQUIRE(a.proj && a.conv_w && a.q_norm && a.k_norm && a.ring && a.q && a.cache && a.rot && a.d_past && m.proj && m.state && m.i_bias && m.f_bias &&
                     (a.S == 1 ? m.out && m.norm : m.gates != nullptr), MYNN_ERR_INVALID, "parallel prepare: null operand");
    const ParallelDims &d = a.d;
    MYNN_REQUIRE(recurrent_dim_supported(d.rdp), MYNN_ERR_UNSUPPORTED, "matrix memory: key dimension %d", d.rd);
    const dim3 grid((unsigned)(2 * a.B * a.S + a.B * d.R));
    const size_t row = (size_t)std::max(d.H, d.G) * d.dimp * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        if (a.S > 1) {
            auto kernel = parallel_prepare_kernel<T, false, 8, 4>;
            int rc = raise_lds(kernel, row);
            if (rc) return rc;
            MYNN_LAUNCH(kernel, grid, dim3(256), row, s, a, m);
            return launch_status("parallel_prepare_kernel");
        }
        return dispatch_columns(d.rdp, [&](auto lc, auto rp) {
            constexpr int LC = decltype(lc)::value, RP = decltype(rp)::value;
            auto kernel = parallel_prepare_kernel<T, true, LC, RP>;
            const size_t lds = std::max(row, (size_t)(2 * LC * RP + d.rvp + 4) * 4);
            int rc = raise_lds(kernel, lds);
            if (rc) return rc;
            MYNN_LAUNCH(kernel, grid, dim3(kStepThreads), lds, s, a, m);
            return launch_status("parallel_prepare_kernel");
        });
    });
}

// ---- several tokens: rows at a time -------------------------------------------------------------------------------------
template <typename T> __global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaParams p) {
    extern __shared__ __align__(16) float buf[];  // q | k of all key heads
    const DeltaDims &d = p.d;
    const int row = blockIdx.x, b = row / p.S, s = row % p.S, past = *p.d_past, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const float *proj = p.proj + (size_t)row * d.n_in(), *ring = p.state + (size_t)b * p.state_stride + d.st_ring();
    for (int ch = tid * 4; ch < d.conv(); ch += 1024) {
        const float4 y = silu4(short_conv4(p.conv_w, proj, d.n_in(), ring, ch, d.conv(), d.taps, s, past));
        *(float4 *)(ch < d.col_v() ? buf + ch : p.v + (size_t)row * d.H * d.vp + ch - d.col_v()) = y;
    }
    for (int h = tid; h < d.H; h += 256) p.beta[(size_t)row * d.H + h] = sigmoidf(proj[d.col_b() + h]);
    for (int i = tid; i < d.low(); i += 256) Elem<T>::st((T *)p.low, (size_t)row * d.low() + i, proj[d.col_low() + i]);
    __syncthreads();
    for (int hk = wave; hk < d.G; hk += 4) {
        const float *q = buf + hk * d.dp, *k = buf + d.col_k() + hk * d.dp;
        float qq = 0.f, kk = 0.f;
        for (int i = lane; i < d.dp; i += 64) {
            qq = fmaf(q[i], q[i], qq);
            kk = fmaf(k[i], k[i], kk);
        }
        const float qn = 1.0f / sqrtf((float)d.d) / sqrtf(wave_sum(qq) + 1e-6f), kn = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
        float *dst = p.qk + (size_t)row * 2 * d.G * d.dp + hk * d.dp;
        for (int i = lane; i < d.dp; i += 64) {
            dst[i] = q[i] * qn;
            dst[d.col_k() + i] = k[i] * kn;
        }
    }
}
int delta_prepare(const DeltaParams &p, int dtype, hipStream_t s) {
    int rc = check_delta(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.qk && p.v && p.beta && p.low, MYNN_ERR_INVALID, "delta prepare: null operand");
    const size_t lds = (size_t)p.d.col_v() * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        int rc2 = raise_lds(delta_prepare_kernel<T>, lds);
        if (rc2) return rc2;
        MYNN_LAUNCH(delta_prepare_kernel<T>, dim3(p.B * p.S), dim3(256), lds, s, p);
        return launch_status("delta_prepare_kernel");
    });
}

// ---- the recurrence, a block of kBlock tokens at a time -----------------------------------------------------------------
constexpr int kBlock = 16;
static_assert(kBlock == kRecurrentBlock, "what the buffers are laid out for");
// operands of block n of (sequence, head) x: [x * nb + n] of each array
struct BlockOperands {
    float *kt, *qt, *kh, *gam, *T, *B;  // [16][KD], [16][KD], [KD][16], [KD], [16][16], [16][16]
};
__device__ __host__ inline BlockOperands block_operands(float *base, size_t blocks, int KD, bool delta) {
    BlockOperands o;
    o.qt = base;
    o.kh = o.qt + blocks * kBlock * KD;
    o.gam = o.kh + blocks * kBlock * KD;
    o.B = o.gam + blocks * KD;
    o.T = o.B + blocks * kBlock * kBlock;
    o.kt = o.T + (delta ? blocks * kBlock * kBlock : 0);
    return o;
}
size_t recurrent_block_floats(int B, int S, int H, int dp, bool delta) {
    const size_t blocks = (size_t)B * H * ((S + kBlock - 1) / kBlock);
    const int KD = recurrent_keys(dp);
    return blocks * ((size_t)(delta ? 3 : 2) * kBlock * KD + KD + (delta ? 2 : 1) * kBlock * kBlock);
}

// G q (and G k) of every token, the keys carried to the block's end, G of the whole block; thread per key channel.
// q, k, g in LDS [16][ldl]; carry(t): what a key of token t is multiplied by
template <bool DELTA, typename Decay, typename Put>
__device__ inline void block_vectors(const BlockOperands &o, size_t blk, int KD, const float *q, const float *k, int ldl, Decay &&decay, Put &&put) {
    for (int c = threadIdx.x; c < KD; c += 256) {
        float G = 1.f;
#pragma unroll
        for (int j = 0; j < kBlock; j++) {
            G *= decay(j, c);
            o.qt[(blk * kBlock + j) * KD + c] = q[j * ldl + c] * G;
            if constexpr (DELTA) o.kt[(blk * kBlock + j) * KD + c] = k[j * ldl + c] * G;
        }
        o.gam[blk * KD + c] = G;
        float w[kBlock], R = 1.f;
#pragma unroll
        for (int i = kBlock - 1; i >= 0; i--) {
            w[i] = k[i * ldl + c] * put(i) * R;
            R *= decay(i, c);
        }
#pragma unroll
        for (int i = 0; i < kBlock; i += 4) *(float4 *)(o.kh + (blk * KD + c) * kBlock + i) = *(const float4 *)(w + i);
    }
}

template <typename T, int KT>  // KD = 64 KT
__global__ __launch_bounds__(256) void delta_blocks_kernel(DeltaParams p, float *base) {
    constexpr int KD = 64 * KT, LDL = KD + 4;
    __shared__ __align__(16) float ks[kBlock * LDL], qs[kBlock * LDL], gs[kBlock * LDL];
    __shared__ float As[kBlock][kBlock + 1], beta[kBlock];
    const DeltaDims &d = p.d;
    const int n = blockIdx.x, h = blockIdx.y, b = blockIdx.z, nb = gridDim.x, hk = h / (d.H / d.G), tid = threadIdx.x;
    const size_t blk = ((size_t)b * d.H + h) * nb + n, row0 = (size_t)b * p.S + n * kBlock;
    const int live = min(kBlock, p.S - n * kBlock);
    const BlockOperands o = block_operands(base, (size_t)gridDim.z * d.H * nb, KD, true);
    const float ea = expf(Elem<T>::ld((const T *)p.a_log, h));
    for (int i = tid; i < kBlock * KD / 4; i += 256) {
        const int t = i / (KD / 4), c = i % (KD / 4) * 4;
        // (tokens past the portion: no key, no query, no decay; channels past the head: nothing)
        float4 k = float4{0.f, 0.f, 0.f, 0.f}, q = k, g = float4{1.f, 1.f, 1.f, 1.f};
        if (t < live && c < d.dp) {
            const float *src = p.qk + (row0 + t) * 2 * d.G * d.dp + hk * d.dp + c;
            q = *(const float4 *)src;
            k = *(const float4 *)(src + d.col_k());
            const float4 a = *(const float4 *)(p.dec + (row0 + t) * d.n_low() + h * d.dp + c);
            const float f[4] = {a.x, a.y, a.z, a.w};
            float *gv = (float *)&g;
#pragma unroll
            for (int e = 0; e < 4; e++) gv[e] = expf(-ea * softplusf(f[e] + Elem<T>::ld((const T *)p.dt_bias, h * d.dp + c + e)));
        }
        *(float4 *)(ks + t * LDL + c) = k;
        *(float4 *)(qs + t * LDL + c) = q;
        *(float4 *)(gs + t * LDL + c) = g;
    }
    if (tid < kBlock) beta[tid] = tid < live ? p.beta[(row0 + tid) * d.H + h] : 0.f;
    __syncthreads();
    // A and B: thread = (earlier token i, sixteenth of the channels)
    {
        const int i = tid >> 4, sl = tid & 15;
        float w[4 * KT];
        float *Bm = o.B + blk * kBlock * kBlock;
        float own = 0.f;
#pragma unroll
        for (int P = 0; P < KT; P++) {
            *(float4 *)(w + 4 * P) = *(const float4 *)(ks + i * LDL + P * 64 + sl * 4);
            const float4 q = *(const float4 *)(qs + i * LDL + P * 64 + sl * 4);
            own = fmaf(w[4 * P], q.x, fmaf(w[4 * P + 1], q.y, fmaf(w[4 * P + 2], q.z, fmaf(w[4 * P + 3], q.w, own))));
        }
        own = group_sum<16>(own);
        if (sl <= i) Bm[sl * kBlock + i] = sl == i ? own : 0.f;  // (row sl, column i: nothing above the diagonal)
        for (int j = i + 1; j < kBlock; j++) {
            float a = 0.f, c = 0.f;
#pragma unroll
            for (int P = 0; P < KT; P++) {
                const float4 g = *(const float4 *)(gs + j * LDL + P * 64 + sl * 4), k = *(const float4 *)(ks + j * LDL + P * 64 + sl * 4);
                const float4 q = *(const float4 *)(qs + j * LDL + P * 64 + sl * 4);
                w[4 * P] *= g.x; w[4 * P + 1] *= g.y; w[4 * P + 2] *= g.z; w[4 * P + 3] *= g.w;
                a = fmaf(w[4 * P], k.x, fmaf(w[4 * P + 1], k.y, fmaf(w[4 * P + 2], k.z, fmaf(w[4 * P + 3], k.w, a))));
                c = fmaf(w[4 * P], q.x, fmaf(w[4 * P + 1], q.y, fmaf(w[4 * P + 2], q.z, fmaf(w[4 * P + 3], q.w, c))));
            }
            a = group_sum<16>(a);
            c = group_sum<16>(c);
            if (sl == 0) {
                As[j][i] = a;
                Bm[j * kBlock + i] = c;
            }
        }
    }
    block_vectors<true>(o, blk, KD, qs, ks, LDL, [&](int t, int c) { return gs[t * LDL + c]; }, [](int) { return 1.f; });
    __syncthreads();
    // T = (1 + diag(beta) A)^-1 diag(beta), a column per thread
    if (tid < kBlock) {
        float x[kBlock];
#pragma unroll
        for (int j = 0; j < kBlock; j++) {
            float s = j == tid ? 1.f : 0.f;
#pragma unroll
            for (int i = 0; i < j; i++) s = i >= tid ? fmaf(-As[j][i], x[i], s) : s;
            x[j] = beta[j] * s;
            o.T[(blk * kBlock + j) * kBlock + tid] = x[j];
        }
    }
}

template <int KT>
__global__ __launch_bounds__(256) void memory_blocks_kernel(MemoryParams p, float *base) {
    constexpr int KD = 64 * KT, LDL = KD + 4;
    __shared__ __align__(16) float ks[kBlock * LDL], qs[kBlock * LDL];
    __shared__ float keep[kBlock], put[kBlock];
    const ParallelDims &d = p.d;
    const int n = blockIdx.x, h = blockIdx.y, b = blockIdx.z, nb = gridDim.x, tid = threadIdx.x;
    const size_t blk = ((size_t)b * d.R + h) * nb + n, row0 = (size_t)b * p.S + n * kBlock;
    const int live = min(kBlock, p.S - n * kBlock);
    const BlockOperands o = block_operands(base, (size_t)gridDim.z * d.R * nb, KD, false);
    for (int i = tid; i < kBlock * KD / 4; i += 256) {
        const int t = i / (KD / 4), c = i % (KD / 4) * 4;
        float4 k = float4{0.f, 0.f, 0.f, 0.f}, q = k;
        if (t < live && c < d.rdp) {
            const float *src = p.proj + (row0 + t) * d.n_in() + h * d.rdp + c;
            q = *(const float4 *)(src + d.mem_q());
            k = *(const float4 *)(src + d.mem_k());
            q.x *= p.q_scale; q.y *= p.q_scale; q.z *= p.q_scale; q.w *= p.q_scale;
        }
        *(float4 *)(ks + t * LDL + c) = k;
        *(float4 *)(qs + t * LDL + c) = q;
    }
    if (tid < kBlock) {
        const float *g = p.gates + ((row0 + min(tid, live - 1)) * d.R + h) * 4;
        keep[tid] = tid < live ? g[0] : 1.f;
        put[tid] = tid < live ? g[1] : 0.f;
    }
    __syncthreads();
    {
        const int j = tid >> 4, i = tid & 15;
        float a = 0.f;
#pragma unroll 8
        for (int c = 0; c < KD; c += 4) {
            const float4 q = *(const float4 *)(qs + j * LDL + c), k = *(const float4 *)(ks + i * LDL + c);
            a = fmaf(q.x, k.x, fmaf(q.y, k.y, fmaf(q.z, k.z, fmaf(q.w, k.w, a))));
        }
        a = i <= j ? a * put[i] : 0.f;
        for (int t = i + 1; t <= j; t++) a *= keep[t];
        o.B[(blk * kBlock + j) * kBlock + i] = a;
    }
    block_vectors<false>(o, blk, KD, qs, ks, LDL, [&](int t, int) { return keep[t]; }, [&](int t) { return put[t]; });
}

struct RecurrenceParams {
    int S, H, dp, ncol, nv;              // ncol: state columns, the first nv of them have a value (else 1)
    const float *v;                      // row * ldv + h * vp + column
    long ldv;
    int vp;
    float *base;                         // block operands
    float *state;
    long state_stride;
    float *o;                            // [row][H][op]
    int op;
    const int32_t *d_past;
};

// Sixteen state columns of a head per workgroup; wave w holds key channels 16 TW w .. of them as TW accumulator tiles of
// v_mfma_f32_16x16x4_f32 (lane (quad, c): channels 4 quad .. + 3 of a tile, column c).  An accumulator register is at the
// same time the second operand of the next product, over the four channels 4 quad + i.
template <bool DELTA, int TW>
__global__ __launch_bounds__(256, 1) void recurrence_kernel(RecurrenceParams p) {
    constexpr int KD = 64 * TW;
    __shared__ __align__(16) float4 part[2][4][2][64];
    typedef float f4_t __attribute__((ext_vector_type(4)));
    const int h = blockIdx.x, c0 = blockIdx.y * 16, b = blockIdx.z, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, quad = lane >> 4;
    const int nb = (p.S + kBlock - 1) / kBlock, col = c0 + c16, k0 = wave * 16 * TW;
    const BlockOperands op = block_operands(p.base, (size_t)gridDim.z * p.H * nb, KD, DELTA);
    const size_t blk0 = ((size_t)b * p.H + h) * nb, row0 = (size_t)b * p.S;
    float *at = p.state + (size_t)b * p.state_stride + ((size_t)h * p.ncol + min(col, p.ncol - 1)) * p.dp;
    const bool fresh = *p.d_past == 0;
    f4_t S[TW];
#pragma unroll
    for (int t = 0; t < TW; t++) {
        const int c = k0 + 16 * t + 4 * quad;
        S[t] = f4_t{0.f, 0.f, 0.f, 0.f};
        if (!fresh && c < p.dp) S[t] = *(const f4_t *)(at + c);
    }
    struct Block {
        f4_t qt[TW], kt[DELTA ? TW : 1], kh[TW], gam[TW], B, T;
        float v[4];
    };
    // (a uniform base and a 32-bit offset of the lane per load, no branches: the waits then count loads exactly)
    const unsigned at_row = (unsigned)(c16 * KD + k0 + 4 * quad), at_key = (unsigned)((k0 + c16) * kBlock + 4 * quad), at_tok = (unsigned)(c16 * kBlock + 4 * quad);
    const bool has_value = col < p.nv;
    const float *values = p.v + row0 * p.ldv + h * p.vp;
    const unsigned vcol = (unsigned)min(col, p.nv - 1);
    auto request = [&](Block &x, int n) {
        const int nn = min(n, nb - 1);
        const size_t blk = blk0 + nn;
        const float *qt = op.qt + blk * kBlock * KD, *kt = op.kt + blk * kBlock * KD, *kh = op.kh + blk * kBlock * KD, *gam = op.gam + blk * KD;
#pragma unroll
        for (int t = 0; t < TW; t++) {
            x.qt[t] = *(const f4_t *)(qt + at_row + 16 * t);
            if constexpr (DELTA) x.kt[t] = *(const f4_t *)(kt + at_row + 16 * t);
            x.kh[t] = *(const f4_t *)(kh + at_key + 16 * t * kBlock);
            x.gam[t] = *(const f4_t *)(gam + k0 + 16 * t + 4 * quad);
        }
        x.B = *(const f4_t *)(op.B + blk * kBlock * kBlock + at_tok);
        if constexpr (DELTA) x.T = *(const f4_t *)(op.T + blk * kBlock * kBlock + at_tok);
#pragma unroll
        for (int i = 0; i < 4; i++) x.v[i] = values[(size_t)min(nn * kBlock + 4 * quad + i, p.S - 1) * p.ldv + vcol];
    };
    auto step = [&](const Block &x, int n) {
        f4_t pq = {0.f, 0.f, 0.f, 0.f}, pk = pq;
#pragma unroll
        for (int t = 0; t < TW; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                pq = __builtin_amdgcn_mfma_f32_16x16x4f32(x.qt[t][i], S[t][i], pq, 0, 0, 0);
                if constexpr (DELTA) pk = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kt[t][i], S[t][i], pk, 0, 0, 0);
            }
        float4(*my)[64] = part[n & 1][wave];
        my[0][lane] = __builtin_bit_cast(float4, pq);
        if constexpr (DELTA) my[1][lane] = __builtin_bit_cast(float4, pk);
#pragma unroll
        for (int t = 0; t < TW; t++) S[t] *= x.gam[t];
        __syncthreads();  // (the other half of `part` was read before the barrier of the block before)
        f4_t u, val;
#pragma unroll
        for (int i = 0; i < 4; i++) val[i] = has_value ? x.v[i] : 1.f;
        if constexpr (DELTA) {
            f4_t sum[4];
#pragma unroll
            for (int w = 0; w < 4; w++) sum[w] = __builtin_bit_cast(f4_t, part[n & 1][w][1][lane]);
            const f4_t r = val - ((sum[0] + sum[1]) + (sum[2] + sum[3]));
            u = f4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < 4; i++) u = __builtin_amdgcn_mfma_f32_16x16x4f32(x.T[i], r[i], u, 0, 0, 0);
        } else u = val;
#pragma unroll
        for (int t = 0; t < TW; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kh[t][i], u[i], S[t], 0, 0, 0);
        if (wave == (n & 3)) {
            f4_t sum[4];
#pragma unroll
            for (int w = 0; w < 4; w++) sum[w] = __builtin_bit_cast(f4_t, part[n & 1][w][0][lane]);
            f4_t out = (sum[0] + sum[1]) + (sum[2] + sum[3]);
#pragma unroll
            for (int i = 0; i < 4; i++) out = __builtin_amdgcn_mfma_f32_16x16x4f32(x.B[i], u[i], out, 0, 0, 0);
            if (col < p.ncol)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int t = n * kBlock + 4 * quad + i;
                    if (t < p.S) p.o[((row0 + t) * p.H + h) * p.op + col] = out[i];
                }
        }
    };
    // the operands of the next AHEAD - 1 blocks are on their way while one is worked on
    constexpr int AHEAD = TW <= 2 ? 4 : TW <= 4 ? 3 : 2;
    Block x[AHEAD];
#pragma unroll
    for (int i = 0; i + 1 < AHEAD; i++) request(x[i], i);
    for (int n0 = 0; n0 < nb; n0 += AHEAD) {
#pragma unroll
        for (int i = 0; i < AHEAD; i++) {
            if (n0 + i >= nb) break;
            request(x[(i + AHEAD - 1) % AHEAD], n0 + i + AHEAD - 1);
            step(x[i], n0 + i);
        }
    }
    if (col < p.ncol)
#pragma unroll
        for (int t = 0; t < TW; t++) {
            const int c = k0 + 16 * t + 4 * quad;
            if (c < p.dp) *(f4_t *)(at + c) = S[t];
        }
}

// f(KT): KD = 64 KT key channels
template <typename F> static int dispatch_keys(int dp, F &&f) {
    using std::integral_constant;
    switch (recurrent_keys(dp)) {
    case 64: return f(integral_constant<int, 1>{});
    case 128: return f(integral_constant<int, 2>{});
    case 256: return f(integral_constant<int, 4>{});
    default: return f(integral_constant<int, 8>{});
    }
}
template <bool DELTA> static int launch_recurrence(const RecurrenceParams &p, int B, hipStream_t s) {
    MYNN_REQUIRE(p.v && p.base && p.state && p.o && p.d_past && B <= 65535 && recurrent_dim_supported(p.dp), MYNN_ERR_INVALID, "recurrence: bad operand");
    return dispatch_keys(p.dp, [&](auto kt) {
        constexpr int KT = decltype(kt)::value;
        MYNN_LAUNCH((recurrence_kernel<DELTA, KT>), dim3(p.H, (p.ncol + 15) / 16, B), dim3(256), 0, s, p);
        return launch_status("recurrence_kernel");
    });
}
int delta_blocks(const DeltaParams &p, int dtype, hipStream_t s) {
    int rc = check_delta(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.qk && p.dec && p.beta && p.blocks && p.a_log && p.dt_bias && p.d.H <= 65535 && p.B <= 65535, MYNN_ERR_INVALID, "delta blocks: bad operand");
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        return dispatch_keys(p.d.dp, [&](auto kt) {
            constexpr int KT = decltype(kt)::value;
            MYNN_LAUNCH((delta_blocks_kernel<T, KT>), dim3((p.S + kBlock - 1) / kBlock, p.d.H, p.B), dim3(256), 0, s, p, p.blocks);
            return launch_status("delta_blocks_kernel");
        });
    });
}
int delta_recurrence(const DeltaParams &p, hipStream_t s) {
    const DeltaDims &d = p.d;
    RecurrenceParams r{};
    r.S = p.S; r.H = d.H; r.dp = d.dp; r.ncol = r.nv = d.v; r.v = p.v; r.ldv = d.H * d.vp; r.vp = d.vp; r.base = p.blocks;
    r.state = p.state; r.state_stride = p.state_stride; r.o = p.o; r.op = d.vp; r.d_past = p.d_past;
    return launch_recurrence<true>(r, p.B, s);
}
int memory_blocks(const MemoryParams &p, hipStream_t s) {
    MYNN_REQUIRE(p.proj && p.gates && p.blocks && p.S > 0 && p.d.R <= 65535 && p.B <= 65535 && recurrent_dim_supported(p.d.rdp), MYNN_ERR_INVALID, "memory blocks: bad operand");
    return dispatch_keys(p.d.rdp, [&](auto kt) {
        constexpr int KT = decltype(kt)::value;
        MYNN_LAUNCH(memory_blocks_kernel<KT>, dim3((p.S + kBlock - 1) / kBlock, p.d.R, p.B), dim3(256), 0, s, p, p.blocks);
        return launch_status("memory_blocks_kernel");
    });
}
int memory_recurrence(const MemoryParams &p, hipStream_t s) {
    const ParallelDims &d = p.d;
    RecurrenceParams r{};
    r.S = p.S; r.H = d.R; r.dp = d.rdp; r.ncol = d.rv + 1; r.nv = d.rv; r.v = p.proj + d.mem_v(); r.ldv = d.n_in(); r.vp = d.rvp; r.base = p.blocks;
    r.state = p.state; r.state_stride = p.state_stride; r.o = p.o; r.op = pad_to(d.rv + 1, 4); r.d_past = p.d_past;
    return launch_recurrence<false>(r, p.B, s);
}

// ---- head norm, output gate, and the conv ring (its readers have run) -----------------------------------------------
struct HeadOutParams {
    int H, v, vp, op;
    const float *o, *den;        // o [row][H][op]; den: memory gates [row][H][4] (null: none)
    const void *norm;            // T, head h at h * norm_stride
    int norm_stride;
    const float *gate;           // f32 before the sigmoid: row * ld_gate + h * vp
    long ld_gate;
    void *out;                   // T: row * ld_out + h * vp
    long ld_out;
    float scale, eps;
    // ring
    const float *proj;
    long ld_proj;
    float *ring;
    long state_stride;
    int channels, taps, rows, S;
    const int32_t *d_past;
};
template <typename T> __global__ __launch_bounds__(256) void head_out_kernel(HeadOutParams p) {
    const int tid = threadIdx.x;
    if ((int)blockIdx.x >= p.rows) {
        // the portion's last taps - 1 projected values of sequence b, column by column
        const int tail = min(p.taps - 1, p.S), per = (p.channels + 255) / 256, id = blockIdx.x - p.rows, b = id / per, ch = id % per * 256 + tid;
        if (ch >= p.channels) return;
        for (int j = 0; j < tail; j++) {
            const int s = p.S - 1 - j;
            p.ring[(size_t)b * p.state_stride + (size_t)((*p.d_past + s) % p.taps) * p.channels + ch] = p.proj[((size_t)b * p.S + s) * p.ld_proj + ch];
        }
        return;
    }
    // 32 lanes per head; a head of up to 128 values stays in registers
    const int row = blockIdx.x, sub = tid & 31;
    for (int h0 = 0; h0 < p.H; h0 += 8) {
        const int h = min(h0 + (tid >> 5), p.H - 1);  // (the last head again: the same values)
        const float *o = p.o + ((size_t)row * p.H + h) * p.op, *g = p.gate + row * p.ld_gate + h * p.vp;
        const T *nw = (const T *)p.norm + h * p.norm_stride;
        T *out = (T *)p.out + row * p.ld_out + h * p.vp;
        float den = 1.f, ss = 0.f;
        auto row4 = [&](int c) {  // (columns past v: zeros)
            float4 x = *(const float4 *)(o + c);
            float *f = (float *)&x;
#pragma unroll
            for (int e = 0; e < 4; e++) f[e] = c + e < p.v ? f[e] : 0.f;
            return x;
        };
        const int c0 = sub * 4, first = min(c0, p.vp - 4);
        const float4 x0 = row4(first), z0 = *(const float4 *)(g + first);
        Load4<T> w0;
        w0.get(nw + first);
        if (p.den) den = 1.0f / (fmaxf(fabsf(o[p.v]), p.den[((size_t)row * p.H + h) * 4 + 2]) + 1e-6f);
        for (int c = c0; c < p.vp; c += 128) {
            const float4 x = c == c0 ? x0 : row4(c);
            ss = fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, ss))));
        }
        const float inv = 1.0f / sqrtf(group_sum<32>(ss) * den * den / (float)p.v + p.eps) * den * p.scale;
        for (int c = c0; c < p.vp; c += 128) {
            float4 x = c == c0 ? x0 : row4(c);
            const float4 z = c == c0 ? z0 : *(const float4 *)(g + c);
            Load4<T> wl = w0;
            if (c != c0) wl.get(nw + c);
            float w[4];
            wl.widen(w);
            x.x *= inv * w[0] * sigmoidf(z.x); x.y *= inv * w[1] * sigmoidf(z.y); x.z *= inv * w[2] * sigmoidf(z.z); x.w *= inv * w[3] * sigmoidf(z.w);
            store4<T>(out + c, x);
        }
    }
}
static int head_out(const HeadOutParams &p, int B, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.o && p.norm && p.gate && p.out && p.proj && p.ring && p.d_past, MYNN_ERR_INVALID, "head norm: null operand");
    const dim3 grid(p.rows + (p.taps > 1 ? B * ((p.channels + 255) / 256) : 0));
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(head_out_kernel<T>, grid, dim3(256), 0, s, p);
        return launch_status("head_out_kernel");
    });
}
int delta_out(const DeltaParams &p, int dtype, hipStream_t s) {
    const DeltaDims &d = p.d;
    HeadOutParams h{};
    h.H = d.H; h.v = d.v; h.vp = h.op = d.vp; h.o = p.o; h.norm = p.norm; h.gate = p.dec + d.H * d.dp; h.ld_gate = d.n_low();
    h.out = p.out; h.ld_out = d.acols(); h.scale = 1.f; h.eps = p.eps;
    h.proj = p.proj; h.ld_proj = d.n_in(); h.ring = p.state + d.st_ring(); h.state_stride = p.state_stride; h.channels = d.conv(); h.taps = d.taps;
    h.rows = p.B * p.S; h.S = p.S; h.d_past = p.d_past;
    return head_out(h, p.B, dtype, s);
}
int memory_out(const WindowAttnParams &a, const MemoryParams &p, int dtype, hipStream_t s) {
    const ParallelDims &d = p.d;
    HeadOutParams h{};
    h.H = d.R; h.v = d.rv; h.vp = d.rvp; h.op = pad_to(d.rv + 1, 4); h.o = p.o; h.den = p.gates; h.norm = p.norm; h.norm_stride = d.rvp;
    h.gate = p.proj + d.mem_g(); h.ld_gate = d.n_in();
    h.out = (char *)p.out + (size_t)d.qcols() * dtype_size(dtype); h.ld_out = d.acols(); h.scale = p.out_scale; h.eps = p.eps;
    h.proj = p.proj; h.ld_proj = d.n_in(); h.ring = a.ring; h.state_stride = a.state_stride; h.channels = d.conv(); h.taps = d.taps;
    h.rows = p.B * p.S; h.S = p.S; h.d_past = p.d_past;
    return head_out(h, p.B, dtype, s);
}

}  // namespace mynn
