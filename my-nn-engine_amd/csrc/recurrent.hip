// Recurrent mixers (see recurrent.h).  A state column -- one value channel of a head -- is a recurrence of its own given the
// keys, queries and gates, so a head's columns are spread over lanes and workgroups.
//
// One new token: delta_step_kernel / the memory workgroups of parallel_prepare_kernel, one workgroup per head, do everything
// between the two projections; the first state columns are requested before anything else.
// Several tokens: the elementwise parts run over all rows at once, then recurrence_kernel walks the tokens.  A column's key
// channels are spread over LC lanes, RP per lane, in registers; keys, queries and decays of a chunk of tokens come through
// LDS, shared by the waves of a workgroup, with the next chunk in registers meanwhile.
#include <algorithm>
#include <type_traits>

#include "dense_load.h"
#include "recurrent.h"

namespace mynn {

__device__ inline float softplusf(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ inline float siluf(float x) { return x * sigmoidf(x); }

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
    for (int i = tid; i < 2 * KD + d.vp; i += kStepThreads) {
        int ch = -1;
        if (i < KD) ch = i < d.dp ? hk * d.dp + i : -1;
        else if (i < 2 * KD) ch = i - KD < d.dp ? d.col_k() + hk * d.dp + i - KD : -1;
        else ch = d.col_v() + h * d.vp + i - 2 * KD;
        float y = 0.f;
        if (ch >= 0) {
            y = siluf(short_conv(p.conv_w, proj, 0, ring, ch, d.conv(), d.taps, 0, past));
            if (keeps || i >= 2 * KD) ring[(size_t)(past % d.taps) * d.conv() + ch] = proj[ch];
        }
        if (i < 2 * KD) qs[i] = y;  // (ks follows qs)
        else vs[i - 2 * KD] = y;
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
template <typename T> __device__ inline MemoryGates memory_gates(const MemoryParams &p, const float *proj, int r) {
    const float zi = (proj[p.d.mem_i() + r] + Elem<T>::ld((const T *)p.i_bias, r)) / p.cap;
    const float zf = (proj[p.d.mem_f() + r] + Elem<T>::ld((const T *)p.f_bias, r)) / p.cap;
    return MemoryGates{p.cap * tanhf(zi), -softplusf(-p.cap * tanhf(zf))};
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
    const MemoryGates gt = memory_gates<T>(p, proj, head);
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

// Gates of all tokens of a portion, one wave per (sequence, head): input and forget gates one token per lane, the running
// maximum token by token.
template <typename T> __device__ inline void memory_gate_scan(const MemoryParams &p, int head, int b) {
    const ParallelDims &d = p.d;
    const int lane = threadIdx.x & 63;
    float *mx = p.state + (size_t)b * p.state_stride + d.st_max() + head;
    float m = *p.d_past ? *mx : 0.f;
    for (int t0 = 0; t0 < p.S; t0 += 64) {
        const size_t row = (size_t)b * p.S + min(t0 + lane, p.S - 1);
        const MemoryGates gt = memory_gates<T>(p, p.proj + row * d.n_in(), head);
        float before = 0.f, after = 0.f;
        const int n = min(64, p.S - t0);
        for (int j = 0; j < n; j++) {
            const float f = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, gt.forget), j));
            const float i = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, gt.in), j));
            const float mn = fmaxf(f + m, i);
            if (lane == j) {
                before = m;
                after = mn;
            }
            m = mn;
        }
        if (lane < n) *(float4 *)(p.gates + (row * d.R + head) * 4) = float4{expf(gt.forget + before - after), expf(gt.in - after), expf(-after), 0.f};
    }
    if (lane == 0) *mx = m;
}

// workgroups 2 row, 2 row + 1: queries and keys of a row of the attention; then one per (sequence, memory head)
template <typename T, bool STEP, int LC, int RP>
__global__ __launch_bounds__(STEP ? kStepThreads : 256) void parallel_prepare_kernel(WindowAttnParams a, MemoryParams m) {
    constexpr int NT = STEP ? kStepThreads : 256;
    extern __shared__ __align__(16) float sm[];
    __shared__ float red[NT / 64];
    const int rows = a.B * a.S, id = blockIdx.x;
    if (id < 2 * rows) {
        window_prepare_row<T, NT>(a, id >> 1, id & 1, sm, red);
        return;
    }
    const int head = (id - 2 * rows) % a.d.R, b = (id - 2 * rows) / a.d.R;
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
    for (int ch = tid; ch < d.conv(); ch += 256) {
        const float y = siluf(short_conv(p.conv_w, proj, d.n_in(), ring, ch, d.conv(), d.taps, s, past));
        if (ch < d.col_v()) buf[ch] = y;
        else p.v[(size_t)row * d.H * d.vp + ch - d.col_v()] = y;
    }
    float *scal = p.scal + (size_t)row * (d.H + d.G);
    for (int h = tid; h < d.H; h += 256) scal[h] = sigmoidf(proj[d.col_b() + h]);
    for (int i = tid; i < d.low(); i += 256) Elem<T>::st((T *)p.low, (size_t)row * d.low() + i, proj[d.col_low() + i]);
    __syncthreads();
    for (int hk = wave; hk < d.G; hk += 4) {
        const float *q = buf + hk * d.dp, *k = buf + d.col_k() + hk * d.dp;
        float qq = 0.f, kk = 0.f, qk = 0.f;
        for (int i = lane; i < d.dp; i += 64) {
            qq = fmaf(q[i], q[i], qq);
            kk = fmaf(k[i], k[i], kk);
            qk = fmaf(q[i], k[i], qk);
        }
        const float qn = 1.0f / sqrtf((float)d.d) / sqrtf(wave_sum(qq) + 1e-6f), kn = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
        qk = wave_sum(qk) * qn * kn;
        float *dst = p.qk + (size_t)row * 2 * d.G * d.dp + hk * d.dp;
        for (int i = lane; i < d.dp; i += 64) {
            dst[i] = q[i] * qn;
            dst[d.col_k() + i] = k[i] * kn;
        }
        if (lane == 0) scal[d.H + hk] = qk;
    }
}
int delta_prepare(const DeltaParams &p, int dtype, hipStream_t s) {
    int rc = check_delta(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.qk && p.v && p.scal && p.low, MYNN_ERR_INVALID, "delta prepare: null operand");
    const size_t lds = (size_t)p.d.col_v() * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        int rc2 = raise_lds(delta_prepare_kernel<T>, lds);
        if (rc2) return rc2;
        MYNN_LAUNCH(delta_prepare_kernel<T>, dim3(p.B * p.S), dim3(256), lds, s, p);
        return launch_status("delta_prepare_kernel");
    });
}

template <typename T> __global__ __launch_bounds__(256) void delta_decays_kernel(DeltaParams p, size_t total) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= total) return;
    const DeltaDims &d = p.d;
    const int n = d.H * d.dp, c = (int)(i % n);
    float *at = p.dec + i / n * d.n_low() + c;
    const float ea = expf(Elem<T>::ld((const T *)p.a_log, c / d.dp));  // (a head's channels come in fours)
    float4 v = *(const float4 *)at;
    float *f = (float *)&v;
#pragma unroll
    for (int e = 0; e < 4; e++) f[e] = expf(-ea * softplusf(f[e] + Elem<T>::ld((const T *)p.dt_bias, c + e)));
    *(float4 *)at = v;
}
int delta_decays(const DeltaParams &p, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.dec && p.a_log && p.dt_bias, MYNN_ERR_INVALID, "delta decays: null operand");
    const size_t total = (size_t)p.B * p.S * p.d.H * p.d.dp;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(delta_decays_kernel<T>, dim3((unsigned)((total / 4 + 255) / 256)), dim3(256), 0, s, p, total);
        return launch_status("delta_decays_kernel");
    });
}

// ---- the recurrence over tokens -----------------------------------------------------------------------------------------
struct RecurrenceParams {
    int S, H, group, dp, ncol, nv;       // group: heads per key head; ncol: state columns, the first nv of them have a value (else 1)
    const float *q, *k, *v, *g;          // row 0 of each; heads at dp / dp / vp / dp
    long ldq, ldk, ldv, ldg;
    int vp;
    float q_scale;
    const float *scal;                   // delta: [row][H + G]; memory: [row][H][4]
    float *state;
    long state_stride;
    float *o;                            // [row][H][op]
    int op;
    const int32_t *d_past;
};
constexpr int kRecThreads = 256, kRecWaves = 4;

template <bool DELTA, int LC, int RP>
__global__ __launch_bounds__(kRecThreads) void recurrence_kernel(RecurrenceParams p) {
    constexpr int KD = LC * RP, CPW = kRecWaves * 64 / LC, TC = KD <= 32 ? 8 : KD <= 128 ? 16 : KD <= 256 ? 8 : 4, NA = DELTA ? 3 : 2;
    constexpr int NL = (TC * KD / 4 + kRecThreads - 1) / kRecThreads;
    constexpr int NV = (TC * CPW + kRecThreads - 1) / kRecThreads;
    static_assert(TC <= LC && TC <= 64, "a lane per token keeps its output");
    extern __shared__ __align__(16) float sm[];  // [2][NA][TC][KD], [2][TC][CPW], [2][TC][2]
    float *vals = sm + 2 * NA * TC * KD, *sc = vals + 2 * TC * CPW;
    const int h = blockIdx.x, c0 = blockIdx.y * CPW, b = blockIdx.z, hk = h / p.group, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int r = lane % LC, cg = wave * (64 / LC) + lane / LC, col = c0 + cg, q4 = p.dp / 4;
    const size_t row0 = (size_t)b * p.S;
    float *at = p.state + (size_t)b * p.state_stride + ((size_t)h * p.ncol + min(col, p.ncol - 1)) * p.dp;
    Column<LC, RP> S;
    S.load(at, r, p.dp);
    const float *src[3] = {p.q + row0 * p.ldq + hk * p.dp, p.k + row0 * p.ldk + hk * p.dp, DELTA ? p.g + row0 * p.ldg + h * p.dp : nullptr};
    const long ld[3] = {p.ldq, p.ldk, p.ldg};
    int lt[NL], lc4[NL];
#pragma unroll
    for (int i = 0; i < NL; i++) {
        const int idx = tid + i * kRecThreads;
        lt[i] = idx / q4;
        lc4[i] = idx % q4 * 4;
    }
    float4 pre[NA][NL];
    float pv[NV], ps[2];
    auto request = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NL; i++)
            if (lt[i] < TC) {
                const int t = min(t0 + lt[i], p.S - 1);
#pragma unroll
                for (int a = 0; a < NA; a++) pre[a][i] = *(const float4 *)(src[a] + (size_t)t * ld[a] + lc4[i]);
            }
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int idx = tid + i * kRecThreads, t = min(t0 + idx / CPW, p.S - 1), c = c0 + idx % CPW;
            pv[i] = 1.f;
            if (idx < TC * CPW && c < p.nv) pv[i] = p.v[(row0 + t) * p.ldv + h * p.vp + c];
        }
        if (tid < TC) {
            const size_t row = row0 + min(t0 + tid, p.S - 1);
            if constexpr (DELTA) {
                const int G = p.H / p.group;
                ps[0] = p.scal[row * (p.H + G) + h];
                ps[1] = p.scal[row * (p.H + G) + p.H + hk];
            } else {
                ps[0] = p.scal[(row * p.H + h) * 4];
                ps[1] = p.scal[(row * p.H + h) * 4 + 1];
            }
        }
    };
    request(0);
    for (int i = tid; i < 2 * NA * TC * KD; i += kRecThreads) sm[i] = 0.f;  // (channels past dp stay zero)
    S.clear(*p.d_past == 0, r, p.dp);
    __syncthreads();
    for (int t0 = 0, buf = 0; t0 < p.S; t0 += TC, buf ^= 1) {
        float *x = sm + buf * NA * TC * KD, *vb = vals + buf * TC * CPW, *sb = sc + buf * TC * 2;
#pragma unroll
        for (int i = 0; i < NL; i++)
            if (lt[i] < TC)
#pragma unroll
                for (int a = 0; a < NA; a++) *(float4 *)(x + (a * TC + lt[i]) * KD + lc4[i]) = pre[a][i];
#pragma unroll
        for (int i = 0; i < NV; i++)
            if (tid + i * kRecThreads < TC * CPW) vb[tid + i * kRecThreads] = pv[i];
        if (tid < TC) {
            sb[2 * tid] = ps[0];
            sb[2 * tid + 1] = ps[1];
        }
        __syncthreads();  // (the other buffer was read before the barrier of the chunk before)
        if (t0 + TC < p.S) request(t0 + TC);
        float mine = 0.f;
        const int n = min(TC, p.S - t0);
        for (int t = 0; t < n; t++) {
            float q[RP], k[RP], g[RP];
            channels_of<LC, RP>(x + t * KD, r, q);
            channels_of<LC, RP>(x + (TC + t) * KD, r, k);
            const float s0 = sb[2 * t], s1 = sb[2 * t + 1], v = vb[t * CPW + cg];
            float o = 0.f;
            if constexpr (DELTA) {
                channels_of<LC, RP>(x + (2 * TC + t) * KD, r, g);
                float a = 0.f;
#pragma unroll
                for (int j = 0; j < RP; j++) {
                    S.s[j] *= g[j];
                    a = fmaf(S.s[j], k[j], a);
                    o = fmaf(S.s[j], q[j], o);
                }
                a = group_sum<LC>(a);
                o = group_sum<LC>(o);
                const float u = s0 * (v - a);
#pragma unroll
                for (int j = 0; j < RP; j++) S.s[j] = fmaf(k[j], u, S.s[j]);
                o = fmaf(s1, u, o);  // (s1 = q . k: the read-out sees this token's write)
            } else {
                const float pvv = s1 * v;
#pragma unroll
                for (int j = 0; j < RP; j++) {
                    S.s[j] = fmaf(k[j], pvv, s0 * S.s[j]);
                    o = fmaf(S.s[j], q[j], o);
                }
                o = group_sum<LC>(o) * p.q_scale;
            }
            mine = r == t ? o : mine;
        }
        if (r < n && col < p.ncol) p.o[((row0 + t0 + r) * p.H + h) * p.op + col] = mine;
    }
    if (col < p.ncol) S.store(at, r, p.dp);
}

template <bool DELTA> static int launch_recurrence(const RecurrenceParams &p, int B, hipStream_t s) {
    MYNN_REQUIRE(p.q && p.k && p.v && p.scal && p.state && p.o && p.d_past && (!DELTA || p.g) && B <= 65535, MYNN_ERR_INVALID, "recurrence: bad operand");
    return dispatch_columns(p.dp, [&](auto lc, auto rp) {
        constexpr int LC = decltype(lc)::value, RP = decltype(rp)::value, KD = LC * RP, CPW = kRecWaves * 64 / LC;
        constexpr int TC = KD <= 32 ? 8 : KD <= 128 ? 16 : KD <= 256 ? 8 : 4, NA = DELTA ? 3 : 2;
        auto kernel = recurrence_kernel<DELTA, LC, RP>;
        const size_t lds = (size_t)(2 * NA * TC * KD + 2 * TC * CPW + 4 * TC) * 4;
        int rc = raise_lds(kernel, lds);
        if (rc) return rc;
        MYNN_LAUNCH(kernel, dim3(p.H, (p.ncol + CPW - 1) / CPW, B), dim3(kRecThreads), lds, s, p);
        return launch_status("recurrence_kernel");
    });
}
int delta_recurrence(const DeltaParams &p, hipStream_t s) {
    const DeltaDims &d = p.d;
    RecurrenceParams r{};
    r.S = p.S; r.H = d.H; r.group = d.H / d.G; r.dp = d.dp; r.ncol = r.nv = d.v;
    r.q = p.qk; r.k = p.qk + d.col_k(); r.v = p.v; r.g = p.dec;
    r.ldq = r.ldk = 2 * d.G * d.dp; r.ldv = d.H * d.vp; r.ldg = d.n_low();
    r.vp = d.vp; r.q_scale = 1.f; r.scal = p.scal; r.state = p.state; r.state_stride = p.state_stride; r.o = p.o; r.op = d.vp; r.d_past = p.d_past;
    return launch_recurrence<true>(r, p.B, s);
}
int memory_recurrence(const MemoryParams &p, hipStream_t s) {
    const ParallelDims &d = p.d;
    RecurrenceParams r{};
    r.S = p.S; r.H = d.R; r.group = 1; r.dp = d.rdp; r.ncol = d.rv + 1; r.nv = d.rv;
    r.q = p.proj + d.mem_q(); r.k = p.proj + d.mem_k(); r.v = p.proj + d.mem_v();
    r.ldq = r.ldk = r.ldv = d.n_in(); r.vp = d.rvp; r.q_scale = p.q_scale; r.scal = p.gates; r.state = p.state; r.state_stride = p.state_stride;
    r.o = p.o; r.op = pad_to(d.rv + 1, 4); r.d_past = p.d_past;
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
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
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
    const int row = blockIdx.x;
    for (int h = wave; h < p.H; h += 4) {
        const float *o = p.o + ((size_t)row * p.H + h) * p.op;
        float den = 1.f, ss = 0.f;
        if (p.den) den = 1.0f / (fmaxf(fabsf(o[p.v]), p.den[((size_t)row * p.H + h) * 4 + 2]) + 1e-6f);
        for (int c = lane; c < p.v; c += 64) {
            const float x = o[c] * den;
            ss = fmaf(x, x, ss);
        }
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)p.v + p.eps) * den;
        const T *nw = (const T *)p.norm + h * p.norm_stride;
        const float *g = p.gate + row * p.ld_gate + h * p.vp;
        T *out = (T *)p.out + row * p.ld_out + h * p.vp;
        for (int c = lane; c < p.vp; c += 64) Elem<T>::st(out, c, c < p.v ? o[c] * inv * Elem<T>::ld(nw, c) * sigmoidf(g[c]) * p.scale : 0.f);
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
