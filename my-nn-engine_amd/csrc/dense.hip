// Linears over weights in the storage type, with the row operators around them, for executors with a 32-bit residual
// stream (declared in dense.h).
//
// One row (decode): dense_gemv_kernel streams the weights once with 16-byte loads, R rows per wave; the workgroup's first
// weights are on their way while it stages the activation row in LDS as f32.  What comes before the linear rides in
// that staging: x' = x + rms_norm(y) * wb of the sublayer before (every workgroup makes the row itself, one of them stores
// x') and the norm in front of this one, so a layer needs no launch for its norms and residual sums.
// Many rows (prefill): residual_norm_rows does the same as one pass per row, and the products run on the matrix cores:
// 16-bit types through gemm_nt_mfma, f32 through gemm_nt_f32_kernel (v_mfma_f32_32x32x2_f32: full f32 products).
#include "dense.h"
#include "dense_load.h"
#include "mfma.h"

namespace mynn {

// ---- weight packing ---------------------------------------------------------------------------------------------------
template <typename T> __global__ void pack_blocks_kernel(PackBlocks p, size_t total) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= total) return;
    const int C = p.CB * p.cols;
    const int c = (int)(i % C);
    const int rr = (int)(i / C);
    const int h = rr / p.rows, j = rr % p.rows;
    int dr = p.dst_row0 + h * p.dst_rs + j;
    if (p.group) dr = (dr / p.group) * 2 * p.group + p.which * p.group + dr % p.group;
    const int sr = p.src_row0 + h * p.src_rs + j;
    const int cb = c / p.cols, cc = c % p.cols;
    ((T *)p.dst)[(size_t)dr * p.ldd + p.dst_col0 + cb * p.dst_cs + cc] = ((const T *)p.src)[(size_t)sr * p.lds + cb * p.src_cs + cc];
}
int pack_blocks(const PackBlocks &p, int dtype, hipStream_t s) {
    const size_t total = (size_t)p.H * p.rows * p.CB * p.cols;
    const dim3 grid((unsigned)((total + 255) / 256));
    if (dtype == MYNN_F32) MYNN_LAUNCH(pack_blocks_kernel<float>, grid, dim3(256), 0, s, p, total);
    else MYNN_LAUNCH(pack_blocks_kernel<uint16_t>, grid, dim3(256), 0, s, p, total);
    return launch_status("pack_blocks_kernel");
}

template <typename T> __global__ void pack_taps_kernel(PackTaps p, int total) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= total) return;
    const int j = i % p.taps, c = i / p.taps;
    p.dst[(size_t)j * p.channels + p.ch0 + c / p.dim * p.dimp + c % p.dim] = Elem<T>::ld((const T *)p.src, i);
}
int pack_taps(const PackTaps &p, int dtype, hipStream_t s) {
    const int total = p.heads * p.dim * p.taps;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(pack_taps_kernel<T>, dim3((total + 255) / 256), dim3(256), 0, s, p, total);
        return launch_status("pack_taps_kernel");
    });
}

// ---- embedding ----------------------------------------------------------------------------------------------------------
__device__ inline size_t history_row(const EmbedParams &p, int b, int r) { return kv_cache_row(p.paging, b, 0, r, 1, p.max_seq); }

template <typename T> __global__ __launch_bounds__(256) void embed_tokens_kernel(EmbedParams p) {
    const int row = blockIdx.x, b = row / p.S, s = row % p.S;
    auto in_vocab = [&](int64_t id) { return id < 0 ? id + p.vocab : id; };
    const int64_t id = in_vocab(p.ids[row]);
    const int pos = *p.d_past + s;
    int64_t pair_row = p.buckets;  // (a sequence's first token)
    if (p.buckets && pos > 0) {
        const int64_t prev = s > 0 ? in_vocab(p.ids[row - 1]) : (int64_t)p.history[history_row(p, b, pos - 1)];
        pair_row = (prev * p.mul_prev + id * p.mul_cur) % p.buckets;
    }
    const int k = blockIdx.y * 256 + threadIdx.x;
    if (k == 0) p.history[history_row(p, b, pos)] = (int32_t)id;
    if (k >= p.ld) return;
    float v = 0.f;
    if (k < p.width) {
        v = Elem<T>::ld((const T *)p.table, (size_t)id * p.width + k);
        if (p.buckets) v += Elem<T>::ld((const T *)p.pair, (size_t)pair_row * p.width + k);
    }
    p.x[(size_t)row * p.ld + k] = v;
    if (p.x0) p.x0[(size_t)row * p.ld + k] = v;
}
int embed_tokens(const EmbedParams &p, int dtype, hipStream_t s) {
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(embed_tokens_kernel<T>, dim3(p.B * p.S, (p.ld + 255) / 256), dim3(256), 0, s, p);
        return launch_status("embed_tokens_kernel");
    });
}

// ---- residual sum and norms of a row, into LDS -----------------------------------------------------------------------
constexpr int kRowThreads = 256, kRowWaves = kRowThreads / kWave;

__device__ inline float row_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < kRowWaves; w++) t += red[w];
    return t;
}

// The row's first kPieces 4-value pieces per thread are requested in one go (a row of up to 4096 values whole); a wider
// row comes in as many rounds.
constexpr int kPieces = 4;
template <typename T> struct RowPieces {
    float4 x[kPieces];
    Load4<T> y[kPieces], wb[kPieces], wa[kPieces];
};
template <typename T>
__device__ inline void row_request(RowPieces<T> &q, const float *x, const T *y, const T *wb, const T *wa, int ld, int base) {
#pragma unroll
    for (int i = 0; i < kPieces; i++) {
        const int k = min(base + (i * kRowThreads + (int)threadIdx.x) * 4, ld - 4);  // (clamped: unconditional loads)
        if (y) { q.y[i].get(y + k); q.wb[i].get(wb + k); }
        q.x[i] = *(const float4 *)(x + k);
        if (wa) q.wa[i].get(wa + k);
    }
}
// act[0, ld) = x' (unnormed) or rms_norm(x') * wa; x_out (may be null) receives x'
template <typename T>
__device__ inline void row_finish(const RowPieces<T> &q, float *act, const float *x, const T *y, const T *wb, const T *wa, float *x_out,
                                  float eps, int width, int ld, float w_add, float y_mul, float *red) {
    constexpr int SPAN = kPieces * kRowThreads * 4;
    const bool one = ld <= SPAN;
    float inv_y = 0.f;
    if (y) {
        float ss = 0.f;
        for (int base = 0; base < ld; base += SPAN) {
#pragma unroll
            for (int i = 0; i < kPieces; i++) {
                const int k = base + (i * kRowThreads + (int)threadIdx.x) * 4;
                if (k < ld) {
                    Load4<T> v = q.y[i];
                    if (!one) v.get(y + k);
                    float f[4];
                    v.widen(f);
                    ss = fmaf(f[0], f[0], fmaf(f[1], f[1], fmaf(f[2], f[2], fmaf(f[3], f[3], ss))));
                }
            }
        }
        inv_y = 1.0f / sqrtf(row_sum(ss, red) / (float)width + eps);
    }
    float ss = 0.f;
    for (int base = 0; base < ld; base += SPAN) {
#pragma unroll
        for (int i = 0; i < kPieces; i++) {
            const int k = base + (i * kRowThreads + (int)threadIdx.x) * 4;
            if (k < ld) {
                float4 v = q.x[i];
                if (!one) v = *(const float4 *)(x + k);
                if (y) {
                    Load4<T> yv = q.y[i], wv = q.wb[i];
                    if (!one) { yv.get(y + k); wv.get(wb + k); }
                    float fy[4], fw[4];
                    yv.widen(fy);
                    wv.widen(fw);
#pragma unroll
                    for (int e = 0; e < 4; e++) fw[e] = (fw[e] + w_add) * y_mul;
                    v.x += fy[0] * inv_y * fw[0]; v.y += fy[1] * inv_y * fw[1];
                    v.z += fy[2] * inv_y * fw[2]; v.w += fy[3] * inv_y * fw[3];
                }
                *(float4 *)(act + k) = v;
                if (x_out) *(float4 *)(x_out + k) = v;
                ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
            }
        }
    }
    if (!wa) return;
    const float inv = 1.0f / sqrtf(row_sum(ss, red) / (float)width + eps);
    for (int base = 0; base < ld; base += SPAN) {
#pragma unroll
        for (int i = 0; i < kPieces; i++) {
            const int k = base + (i * kRowThreads + (int)threadIdx.x) * 4;
            if (k < ld) {
                Load4<T> wv = q.wa[i];
                if (!one) wv.get(wa + k);
                float fw[4];
                wv.widen(fw);
                float4 v = *(float4 *)(act + k);
                v.x *= inv * (fw[0] + w_add); v.y *= inv * (fw[1] + w_add); v.z *= inv * (fw[2] + w_add); v.w *= inv * (fw[3] + w_add);
                *(float4 *)(act + k) = v;
            }
        }
    }
}

template <typename T, int PRO>
__global__ __launch_bounds__(kRowThreads) void residual_norm_rows_kernel(T *act_out, ResidualNorm r, int first, int stride) {
    extern __shared__ __align__(16) float act[];
    __shared__ float red[kRowWaves];
    const size_t row = (size_t)first + (size_t)blockIdx.x * stride, at = row * r.ld;
    const float *x = r.x + at;
    const T *y = r.y ? (const T *)r.y + at : nullptr;
    const T *wa = PRO == PRO_RESIDUAL_NORM ? (const T *)r.wa : nullptr;
    RowPieces<T> q;
    row_request<T>(q, x, y, (const T *)r.wb, wa, r.ld, 0);
    row_finish<T>(q, act, x, y, (const T *)r.wb, wa, r.x_out ? r.x_out + at : nullptr, r.eps, r.width, r.ld, r.w_add, r.y_mul, red);
    T *out = act_out + (size_t)blockIdx.x * r.ld * (PRO == PRO_RESIDUAL_CONCAT ? 2 : 1);
    for (int k = threadIdx.x * 4; k < r.ld; k += kRowThreads * 4) {  // (a thread reads back what it wrote)
        store4<T>(out + k, *(const float4 *)(act + k));
        if constexpr (PRO == PRO_RESIDUAL_CONCAT) store4<T>(out + r.ld + k, *(const float4 *)(r.x0 + at + k));
    }
}

static int check_row(const ResidualNorm &r, int pro) {
    MYNN_REQUIRE(r.x && (!r.y || r.wb) && r.ld % 64 == 0 && r.width > 0 && r.width <= r.ld, MYNN_ERR_INVALID, "residual norm: bad row");
    MYNN_REQUIRE(pro != PRO_RESIDUAL_NORM || r.wa, MYNN_ERR_INVALID, "residual norm: no norm weights");
    MYNN_REQUIRE(pro != PRO_RESIDUAL_CONCAT || r.x0, MYNN_ERR_INVALID, "residual norm: nothing to append");
    return 0;
}
constexpr size_t kRowLdsMax = 152 * 1024;
template <typename K> static int allow_lds(K kernel) {
    MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kRowLdsMax));
    return 0;
}

int residual_norm_rows(void *act, const ResidualNorm &r, int pro, int first, int stride, int count, int dtype, hipStream_t s) {
    int rc = check_row(r, pro);
    if (rc) return rc;
    const size_t lds = (size_t)r.ld * 4;
    MYNN_REQUIRE(lds <= kRowLdsMax, MYNN_ERR_UNSUPPORTED, "residual norm: rows of %d values", r.ld);
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        auto go = [&](auto kernel) {
            if (lds > 60 * 1024) { int rc2 = allow_lds(kernel); if (rc2) return rc2; }
            MYNN_LAUNCH(kernel, dim3(count), dim3(kRowThreads), lds, s, (T *)act, r, first, stride);
            return launch_status("residual_norm_rows_kernel");
        };
        if (pro == PRO_RESIDUAL) return go(residual_norm_rows_kernel<T, PRO_RESIDUAL>);
        return pro == PRO_RESIDUAL_CONCAT ? go(residual_norm_rows_kernel<T, PRO_RESIDUAL_CONCAT>) : go(residual_norm_rows_kernel<T, PRO_RESIDUAL_NORM>);
    });
}

// best (value, index) of a workgroup's threads, in thread 0
__device__ inline void workgroup_best(float &bv, int &bi, GreedyCand *best) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
        const float ov = __shfl_xor(bv, off, kWave);
        const int oi = __shfl_xor(bi, off, kWave);
        if (oi >= 0) argmax_take(bv, bi, ov, oi);
    }
    if ((threadIdx.x & 63) == 0) best[threadIdx.x >> 6] = GreedyCand{bv, bi};
    __syncthreads();
    if (threadIdx.x == 0)
        for (int w = 1; w < kRowWaves; w++)
            if (best[w].index >= 0) argmax_take(bv, bi, best[w].value, best[w].index);
}

// ---- one-row linear -----------------------------------------------------------------------------------------------------
// A wave's row group: R rows; GEGLU: R / 2 gate rows and the R / 2 up rows 32 further on.
template <typename T, int R, int PRO, int STORE>
__global__ __launch_bounds__(kRowThreads) void dense_gemv_kernel(const T *w, const void *act_in, int N, int K, int groups, int total_waves,
                                                                 void *out, const float *scale, ResidualNorm r, GreedyCand *cand) {
    constexpr int E = 16 / (int)sizeof(T);  // weights per 16-byte load
    constexpr int UN = sizeof(T) == 2 ? 4 : 4;
    extern __shared__ __align__(16) float act[];  // [K]
    __shared__ float red[kRowWaves];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int nch = K / E;
    auto row_of = [&](int g, int i) {
        if constexpr (STORE == DENSE_GEGLU) {
            const int o = g * (R / 2) + i % (R / 2);
            return (o >> 5) * 64 + (o & 31) + (i >= R / 2 ? 32 : 0);
        } else return min(g * R + i, N - 1);
    };
    U4 wv[R][UN];
    auto load = [&](int g, int c0) {
#pragma unroll
        for (int i = 0; i < R; i++) {
            const U4 *p = (const U4 *)(w + (size_t)row_of(g, i) * K);
#pragma unroll
            for (int u = 0; u < UN; u++) wv[i][u] = __builtin_nontemporal_load(&p[min(c0 + u * 64 + lane, nch - 1)]);
        }
    };
    int g = blockIdx.x * kRowWaves + wave;
    // the activation is requested first (loads return in order), then the first weights, then the activation is staged
    if constexpr (PRO == PRO_ROWS) {
        Load4<T> a[kPieces];
        const T *ap = (const T *)act_in;
#pragma unroll
        for (int i = 0; i < kPieces; i++) a[i].get(ap + min((i * kRowThreads + (int)threadIdx.x) * 4, K - 4));
        load(min(g, groups - 1), 0);
#pragma unroll
        for (int i = 0; i < kPieces; i++) {
            const int k = (i * kRowThreads + (int)threadIdx.x) * 4;
            if (k < K) {
                float4 f;
                a[i].widen((float *)&f);
                *(float4 *)(act + k) = f;
            }
        }
        for (int k = (kPieces * kRowThreads + (int)threadIdx.x) * 4; k < K; k += kRowThreads * 4) {
            Load4<T> v;
            v.get(ap + k);
            float4 f;
            v.widen((float *)&f);
            *(float4 *)(act + k) = f;
        }
    } else {
        const T *y = (const T *)r.y, *wb = (const T *)r.wb, *wa = PRO == PRO_RESIDUAL_NORM ? (const T *)r.wa : nullptr;
        RowPieces<T> q;
        row_request<T>(q, r.x, y, wb, wa, r.ld, 0);
        load(min(g, groups - 1), 0);
        row_finish<T>(q, act, r.x, y, wb, wa, blockIdx.x == 0 ? r.x_out : nullptr, r.eps, r.width, r.ld, r.w_add, r.y_mul, red);
        if constexpr (PRO == PRO_RESIDUAL_CONCAT)
            for (int k = threadIdx.x * 4; k < r.ld; k += kRowThreads * 4) *(float4 *)(act + r.ld + k) = *(const float4 *)(r.x0 + k);
    }
    __syncthreads();

    float bv = -INFINITY;  // this lane's best output so far (cand)
    int bi = -1;
    bool first = true;
    for (; g < groups; g += total_waves) {
        float acc[R];
#pragma unroll
        for (int i = 0; i < R; i++) acc[i] = 0.f;
        for (int c0 = 0; c0 < nch; c0 += 64 * UN) {
            if (!first) load(g, c0);
            first = false;
#pragma unroll
            for (int u = 0; u < UN; u++) {
                const int c = c0 + u * 64 + lane;
                if (c < nch) {
                    float a[E];
#pragma unroll
                    for (int e = 0; e < E; e += 4) *(float4 *)(a + e) = *(const float4 *)(act + c * E + e);
#pragma unroll
                    for (int i = 0; i < R; i++) {
                        float f[E];
                        widen16b<T>(wv[i][u], f);
#pragma unroll
                        for (int e = 0; e < E; e++) acc[i] = fmaf(f[e], a[e], acc[i]);
                    }
                }
            }
        }
#pragma unroll
        for (int i = 0; i < R; i++) acc[i] = wave_sum(acc[i]);
        // lane i finishes row i
        if constexpr (STORE == DENSE_GEGLU) {
#pragma unroll
            for (int i = 0; i < R / 2; i++) {
                const int o = g * (R / 2) + i;
                if (lane == i && o < N / 2) Elem<T>::st((T *)out, o, gelu_tanh(acc[i]) * acc[R / 2 + i]);
            }
        } else {
            float mine = acc[0];
#pragma unroll
            for (int i = 1; i < R; i++)
                if (lane == i) mine = acc[i];
            const int n = g * R + lane;
            if (lane < R && n < N) {
                if constexpr (STORE == DENSE_F32) {
                    const float v = scale ? mine * *scale : mine;
                    ((float *)out)[n] = v;
                    argmax_take(bv, bi, v, n);
                } else Elem<T>::st((T *)out, n, mine);
            }
        }
    }
    if constexpr (STORE == DENSE_F32) {
        if (cand) {
            __shared__ GreedyCand best[kRowWaves];
            workgroup_best(bv, bi, best);
            if (threadIdx.x == 0) cand[blockIdx.x] = GreedyCand{bv, bi};
        }
    }
}

// the best of the workgroups' candidates (the last maximum wins), as argmax_rows leaves it
__global__ __launch_bounds__(256) void greedy_pick_kernel(int32_t *out, const GreedyCand *cand, int n, AdvanceState adv) {
    __shared__ GreedyCand best[4];
    int st_step = 0, st_past = 0, st_active = 0;
    int64_t st_pos = 0;
    if (adv.ids && threadIdx.x == 0) {
        st_step = *adv.step;
        st_pos = adv.pos[0];
        st_past = *adv.past;
        st_active = *adv.active;
    }
    float bv = -INFINITY;
    int bi = -1;
    for (int i = threadIdx.x; i < n; i += 256)
        if (cand[i].index >= 0) argmax_take(bv, bi, cand[i].value, cand[i].index);
    workgroup_best(bv, bi, best);
    if (threadIdx.x) return;
    out[0] = bi;
    if (adv.ids) {
        if (st_step < adv.cap) adv.tokens[st_step] = bi;
        *adv.step = st_step + 1;
        adv.ids[0] = bi;
        adv.pos[0] = st_pos + 1;
        *adv.past = st_past + 1;
        *adv.active = st_active + 1;
    }
}
int greedy_pick(int32_t *out, const GreedyCand *cand, int n, AdvanceState adv, hipStream_t s) {
    MYNN_REQUIRE(out && cand && n > 0, MYNN_ERR_INVALID, "greedy pick: bad operand");
    MYNN_LAUNCH(greedy_pick_kernel, dim3(1), dim3(256), 0, s, out, cand, n, adv);
    return launch_status("greedy_pick_kernel");
}

bool dense_gemv_supported(int K) { return K % 64 == 0 && (size_t)K * 4 <= kRowLdsMax; }

template <typename T, int R, int PRO, int STORE>
static int launch_gemv(void *out, const void *act, const ResidualNorm &r, const void *w, int N, int K, const float *scale, hipStream_t s,
                       GreedyCand *cand, int *n_cand) {
    const int groups = STORE == DENSE_GEGLU ? (N / 2 + R / 2 - 1) / (R / 2) : (N + R - 1) / R;
    const size_t lds = (size_t)K * 4;
    const int per_cu = (int)(kRowLdsMax / lds) < 4 ? (int)(kRowLdsMax / lds) : 4;
    const int max_waves = 256 * kRowWaves * per_cu;
    const int passes = (groups + max_waves - 1) / max_waves;
    const int blocks = ((groups + passes - 1) / passes + kRowWaves - 1) / kRowWaves;
    auto kernel = dense_gemv_kernel<T, R, PRO, STORE>;
    if (lds > 60 * 1024) { int rc = allow_lds(kernel); if (rc) return rc; }
    MYNN_LAUNCH(kernel, dim3(blocks), dim3(kRowThreads), lds, s, (const T *)w, act, N, K, groups, blocks * kRowWaves, out, scale, r, cand);
    if (n_cand) *n_cand = blocks;
    return launch_status("dense_gemv_kernel");
}

int dense_gemv(void *out, const void *act, const ResidualNorm *r, int pro, const void *w, int N, int K, int store, const float *scale,
               int dtype, hipStream_t s, GreedyCand *cand, int *n_cand) {
    MYNN_REQUIRE(!cand || store == DENSE_F32, MYNN_ERR_INVALID, "dense gemv: candidates of store %d", store);
    MYNN_REQUIRE(out && w && N > 0 && dense_gemv_supported(K), MYNN_ERR_INVALID, "dense gemv: N=%d K=%d", N, K);
    MYNN_REQUIRE(store != DENSE_GEGLU || N % 64 == 0, MYNN_ERR_INVALID, "dense gemv: %d interleaved gate/up rows", N);
    if (pro == PRO_ROWS) MYNN_REQUIRE(act, MYNN_ERR_INVALID, "dense gemv: null activation");
    else {
        int rc = r ? check_row(*r, pro) : fail(MYNN_ERR_INVALID, "dense gemv: no row");
        if (rc) return rc;
        MYNN_REQUIRE(K == r->ld * (pro == PRO_RESIDUAL_CONCAT ? 2 : 1) && r->x_out != r->x, MYNN_ERR_INVALID, "dense gemv: row of %d for K=%d", r->ld, K);
    }
    const ResidualNorm none{};
    const ResidualNorm &rr = r ? *r : none;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        if (pro == PRO_RESIDUAL_CONCAT) {
            MYNN_REQUIRE(store == DENSE_F32, MYNN_ERR_UNSUPPORTED, "dense gemv: concatenated row with store %d", store);
            return launch_gemv<T, 2, PRO_RESIDUAL_CONCAT, DENSE_F32>(out, act, rr, w, N, K, scale, s, cand, n_cand);
        }
        if (pro == PRO_RESIDUAL) {
            MYNN_REQUIRE(store == DENSE_F32, MYNN_ERR_UNSUPPORTED, "dense gemv: unnormed row with store %d", store);
            return launch_gemv<T, 2, PRO_RESIDUAL, DENSE_F32>(out, act, rr, w, N, K, scale, s, cand, n_cand);
        }
        if (pro == PRO_RESIDUAL_NORM) {
            if (store == DENSE_GEGLU) return launch_gemv<T, 4, PRO_RESIDUAL_NORM, DENSE_GEGLU>(out, act, rr, w, N, K, scale, s, cand, n_cand);
            if (store == DENSE_F32) return launch_gemv<T, 4, PRO_RESIDUAL_NORM, DENSE_F32>(out, act, rr, w, N, K, scale, s, cand, n_cand);
            return launch_gemv<T, 2, PRO_RESIDUAL_NORM, DENSE_T>(out, act, rr, w, N, K, scale, s, cand, n_cand);
        }
        MYNN_REQUIRE(store == DENSE_T, MYNN_ERR_UNSUPPORTED, "dense gemv: plain row with store %d", store);
        return launch_gemv<T, 2, PRO_ROWS, DENSE_T>(out, act, rr, w, N, K, scale, s, cand, n_cand);
    });
}

// ---- many-row linear, f32: 128 x 64 outputs per workgroup, a wave owns 32 rows x 64 columns, K step 16 --------------
typedef float f16acc_t __attribute__((ext_vector_type(16)));
// GROUPED: row tile blockIdx.y multiplies its group's weight (GroupedRows); DENSE_GEGLU then stores silu(gate) * up
template <int STORE, bool GROUPED>
__global__ __launch_bounds__(256) void gemm_nt_f32_kernel(float *out, const float *A, const float *B, int M, int N, int K, const float *scale, GroupedRows gr) {
    constexpr int BK = 16, LD = BK + 4;
    __shared__ __align__(16) float As[128 * LD], Bs[64 * LD];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int m0 = blockIdx.y * 128, n0 = blockIdx.x * 64;
    const int lr = tid >> 2, lc = (tid & 3) * 4;
    if constexpr (GROUPED) {
        const int grp = gr.tile_group[blockIdx.y * 128 / gr.group_rows];
        if (grp < 0) return;
        B += (size_t)grp * gr.group_elems;
    }
    auto a_row = [&](int r) {
        if constexpr (GROUPED) return gr.gather ? max(gr.slot[r], 0) / gr.per_row : r;
        else return min(r, M - 1);
    };
    const float *a0 = A + (size_t)a_row(m0 + lr) * K + lc, *a1 = A + (size_t)a_row(m0 + lr + 64) * K + lc;
    const float *b0 = B + (size_t)min(n0 + lr, N - 1) * K + lc;
    f16acc_t acc[2];
#pragma unroll
    for (int j = 0; j < 2; j++)
#pragma unroll
        for (int e = 0; e < 16; e++) acc[j][e] = 0.f;
    const int fr = lane & 31, fk = lane >> 5;
    for (int k0 = 0; k0 < K; k0 += BK) {
        const float4 va = *(const float4 *)(a0 + k0), vb = *(const float4 *)(a1 + k0), vc = *(const float4 *)(b0 + k0);
        __syncthreads();
        *(float4 *)&As[lr * LD + lc] = va;
        *(float4 *)&As[(lr + 64) * LD + lc] = vb;
        *(float4 *)&Bs[lr * LD + lc] = vc;
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; k += 2) {
            const float a = As[(wave * 32 + fr) * LD + k + fk];
#pragma unroll
            for (int j = 0; j < 2; j++)
                acc[j] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, Bs[(j * 32 + fr) * LD + k + fk], acc[j], 0, 0, 0);
        }
    }
    // lane: column fr of a column tile, rows 8 * (e / 4) + 4 * fk + e % 4
    const float sc = scale ? *scale : 1.f;
#pragma unroll
    for (int e = 0; e < 16; e++) {
        const int row = m0 + wave * 32 + 8 * (e >> 2) + 4 * fk + (e & 3);
        if constexpr (GROUPED) {
            const int as = gr.slot[row];
            if (as < 0) continue;
            if constexpr (STORE == DENSE_GEGLU) {
                const float gate = acc[0][e] * gr.scale[as], up = acc[1][e] * gr.scale[as];
                out[(size_t)row * (N / 2) + n0 / 2 + fr] = gate * sigmoidf(gate) * up;
            } else {
#pragma unroll
                for (int j = 0; j < 2; j++)
                    if (n0 + j * 32 + fr < N) out[(size_t)as * N + n0 + j * 32 + fr] = acc[j][e];
            }
            continue;
        }
        if (row >= M) continue;
        if constexpr (STORE == DENSE_GEGLU) {
            out[(size_t)row * (N / 2) + n0 / 2 + fr] = gelu_tanh(acc[0][e]) * acc[1][e];
        } else {
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const int n = n0 + j * 32 + fr;
                if (n < N) out[(size_t)row * N + n] = acc[j][e] * sc;
            }
        }
    }
}

int dense_gemm(void *out, const void *act, const void *w, int M, int N, int K, int store, const float *scale, int dtype, hipStream_t s) {
    MYNN_REQUIRE(out && act && w && M > 0 && N > 0 && K > 0 && K % 64 == 0, MYNN_ERR_INVALID, "dense gemm: M=%d N=%d K=%d", M, N, K);
    MYNN_REQUIRE(store != DENSE_GEGLU || N % 64 == 0, MYNN_ERR_INVALID, "dense gemm: %d interleaved gate/up rows", N);
    if (dtype != MYNN_F32)
        return gemm_nt_mfma(out, act, w, store == DENSE_F32 ? scale : nullptr, M, N, K, dtype,
                            store == DENSE_GEGLU ? GEMM_GEGLU : store == DENSE_F32 ? GEMM_F32 : GEMM_PLAIN, s);
    const dim3 grid((N + 63) / 64, (M + 127) / 128);
    MYNN_REQUIRE(grid.y <= 65535, MYNN_ERR_UNSUPPORTED, "dense gemm: M=%d", M);
    if (store == DENSE_GEGLU)
        MYNN_LAUNCH((gemm_nt_f32_kernel<DENSE_GEGLU, false>), grid, dim3(256), 0, s, (float *)out, (const float *)act, (const float *)w, M, N, K, scale, GroupedRows{});
    else
        MYNN_LAUNCH((gemm_nt_f32_kernel<DENSE_F32, false>), grid, dim3(256), 0, s, (float *)out, (const float *)act, (const float *)w, M, N, K, scale, GroupedRows{});
    return launch_status("gemm_nt_f32_kernel");
}

int gemm_grouped(void *out, const void *act, const void *wt, const GroupedRows &g, int N, int K, int epi, int dtype, hipStream_t s) {
    MYNN_REQUIRE(out && act && wt && g.tile_group && g.slot && g.per_row > 0 && N > 0 && K > 0 && K % 64 == 0 && g.tiles > 0 && g.tiles <= 65535,
                 MYNN_ERR_INVALID, "grouped gemm: %d tiles, N=%d K=%d", g.tiles, N, K);
    MYNN_REQUIRE(g.gather == (epi == GEMM_SILU) && (epi != GEMM_SILU || (N % 64 == 0 && g.scale)), MYNN_ERR_INVALID, "grouped gemm: store %d of N=%d", epi, N);
    if (dtype == MYNN_BF16) return gemm_grouped_bf16(out, act, wt, g, N, K, epi, s);
    MYNN_REQUIRE(dtype == MYNN_F32, MYNN_ERR_UNSUPPORTED, "grouped gemm: dtype %d", dtype);
    MYNN_REQUIRE(g.group_rows % 128 == 0, MYNN_ERR_INVALID, "grouped gemm: groups of %d rows", g.group_rows);
    const dim3 grid((N + 63) / 64, g.tiles * (g.group_rows / 128));
    MYNN_REQUIRE(grid.y <= 65535, MYNN_ERR_UNSUPPORTED, "grouped gemm: %d tiles", g.tiles);
    if (epi == GEMM_SILU)
        MYNN_LAUNCH((gemm_nt_f32_kernel<DENSE_GEGLU, true>), grid, dim3(256), 0, s, (float *)out, (const float *)act, (const float *)wt, 0, N, K, nullptr, g);
    else
        MYNN_LAUNCH((gemm_nt_f32_kernel<DENSE_F32, true>), grid, dim3(256), 0, s, (float *)out, (const float *)act, (const float *)wt, 0, N, K, nullptr, g);
    return launch_status("gemm_nt_f32_kernel");
}

}  // namespace mynn
