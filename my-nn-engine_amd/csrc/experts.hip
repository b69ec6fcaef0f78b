// Sparse feed-forward (see experts.h).
//
// One row (decode): the router's logits come from the ordinary one-row linear; expert_gateup_row_kernel picks its expert from
// them (every workgroup for itself) and streams that expert's rows, expert_down_row_kernel adds the experts' products up in
// f32.  Several rows: route_rows_kernel scores a few rows per workgroup, sort_kernel lists the assignments expert by expert in
// whole tiles, and the two products run as grouped matrix-core products over that list (gemm_grouped).
#include <algorithm>

#include "dense_load.h"
#include "experts.h"

namespace mynn {

constexpr int kRowT = 256, kRowW = 4;
__device__ inline float silu_of(float z) { return z * sigmoidf(z); }

// Wave-wide: index of the n-th largest of z[0, E) (n < E; of equal ones the first); z is in LDS and loses the ones found.
__device__ inline int take_largest(float *z, int E, int n) {
    const int lane = threadIdx.x & 63;
    int best = 0;
    for (int i = 0; i <= n; i++) {
        float bv = -INFINITY;
        int bi = -1;
        for (int e = lane; e < E; e += 64)
            if (z[e] > bv) {
                bv = z[e];
                bi = e;
            }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) {
            const float ov = __shfl_xor(bv, off, 64);
            const int oi = __shfl_xor(bi, off, 64);
            if (oi >= 0 && (bi < 0 || ov > bv || (ov == bv && oi < bi))) {
                bv = ov;
                bi = oi;
            }
        }
        best = bi < 0 ? 0 : bi;  // (nothing above minus infinity: still an expert)
        if (lane == 0 && i < n) z[best] = -INFINITY;
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt(0): the mark is there before the next search
    }
    return best;
}

// ---- one row ------------------------------------------------------------------------------------------------------------
// R = 4 rows per wave: two gate rows and their up rows, 32 further on
template <typename T>
__global__ __launch_bounds__(kRowT) void expert_gateup_row_kernel(ExpertParams p) {
    constexpr int E16 = 16 / (int)sizeof(T), UN = 4, R = 4;
    extern __shared__ __align__(16) float act[];  // [ld], then the logits [E]
    __shared__ int s_expert;
    __shared__ float s_score;
    float *z = act + p.ld;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, which = blockIdx.y;
    for (int k = tid * 4; k < p.ld; k += kRowT * 4) *(float4 *)(act + k) = *(const float4 *)(p.x + k);
    for (int e = tid; e < p.E; e += kRowT) z[e] = p.logits[e];
    __syncthreads();
    if (wave == 0) {
        const int e = take_largest(z, p.E, which);
        if (lane == 0) {
            s_expert = e;
            s_score = sigmoidf(z[e]);
            if (blockIdx.x == 0) p.chosen[which] = e;
        }
    }
    __syncthreads();
    const float score = s_score;
    const T *w = (const T *)p.gu + (size_t)s_expert * 2 * p.fp * p.ld;
    const int nch = p.ld / E16, groups = p.fp / 2, stride = gridDim.x * kRowW;
    for (int g = blockIdx.x * kRowW + wave; g < groups; g += stride) {
        const int o = g * 2, row = (o >> 5) * 64 + (o & 31);
        const int rows[R] = {row, row + 1, row + 32, row + 33};
        float acc[R] = {0.f, 0.f, 0.f, 0.f};
        for (int c0 = 0; c0 < nch; c0 += 64 * UN) {
            U4 wv[R][UN];
#pragma unroll
            for (int i = 0; i < R; i++)
#pragma unroll
                for (int u = 0; u < UN; u++) wv[i][u] = __builtin_nontemporal_load((const U4 *)(w + (size_t)rows[i] * p.ld) + min(c0 + u * 64 + lane, nch - 1));
#pragma unroll
            for (int u = 0; u < UN; u++) {
                const int c = c0 + u * 64 + lane;
                if (c < nch) {
                    float a[E16];
#pragma unroll
                    for (int e = 0; e < E16; e += 4) *(float4 *)(a + e) = *(const float4 *)(act + c * E16 + e);
#pragma unroll
                    for (int i = 0; i < R; i++) {
                        float f[E16];
                        widen16b<T>(wv[i][u], f);
#pragma unroll
                        for (int e = 0; e < E16; e++) acc[i] = fmaf(f[e], a[e], acc[i]);
                    }
                }
            }
        }
#pragma unroll
        for (int i = 0; i < R; i++) acc[i] = wave_sum(acc[i]) * score;
        if (lane < 2) {
            const float gate = lane ? acc[1] : acc[0], up = lane ? acc[3] : acc[2];
            Elem<T>::st((T *)p.hmid, (size_t)which * p.fp + o + lane, silu_of(gate) * up);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(kRowT) void expert_down_row_kernel(ExpertParams p) {
    constexpr int E16 = 16 / (int)sizeof(T), UN = 4, R = 2;
    extern __shared__ __align__(16) float act[];  // [top][fp]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nch = p.fp / E16, groups = p.ld / R, stride = gridDim.x * kRowW;
    for (int k = tid * 4; k < p.top * p.fp; k += kRowT * 4) {
        Load4<T> v;
        v.get((const T *)p.hmid + k);
        v.widen(act + k);
    }
    __syncthreads();
    for (int g = blockIdx.x * kRowW + wave; g < groups; g += stride) {
        float acc[R] = {0.f, 0.f};
        for (int x = 0; x < p.top; x++) {
            const T *w = (const T *)p.down + ((size_t)p.chosen[x] * p.ld + (size_t)g * R) * p.fp;
            const float *av = act + x * p.fp;
            for (int c0 = 0; c0 < nch; c0 += 64 * UN) {
                U4 wv[R][UN];
#pragma unroll
                for (int i = 0; i < R; i++)
#pragma unroll
                    for (int u = 0; u < UN; u++) wv[i][u] = __builtin_nontemporal_load((const U4 *)(w + (size_t)i * p.fp) + min(c0 + u * 64 + lane, nch - 1));
#pragma unroll
                for (int u = 0; u < UN; u++) {
                    const int c = c0 + u * 64 + lane;
                    if (c < nch) {
                        float a[E16];
#pragma unroll
                        for (int e = 0; e < E16; e += 4) *(float4 *)(a + e) = *(const float4 *)(av + c * E16 + e);
#pragma unroll
                        for (int i = 0; i < R; i++) {
                            float f[E16];
                            widen16b<T>(wv[i][u], f);
#pragma unroll
                            for (int e = 0; e < E16; e++) acc[i] = fmaf(f[e], a[e], acc[i]);
                        }
                    }
                }
            }
        }
#pragma unroll
        for (int i = 0; i < R; i++) acc[i] = wave_sum(acc[i]);
        if (lane < R) Elem<T>::st((T *)p.y, (size_t)g * R + lane, lane ? acc[1] : acc[0]);
    }
}

constexpr size_t kExpertLds = 152 * 1024;
template <typename K> static int raise_lds(K kernel, size_t lds) {
    MYNN_REQUIRE(lds <= kExpertLds, MYNN_ERR_UNSUPPORTED, "experts: rows of %zu bytes", lds);
    if (lds > 60 * 1024) MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kExpertLds));
    return 0;
}
bool expert_row_supported(int ld, int fp, int top) { return (size_t)ld * 4 + 16 * 1024 <= kExpertLds && (size_t)top * fp * 4 <= kExpertLds; }

static int check_experts(const ExpertParams &p) {
    MYNN_REQUIRE(p.gu && p.down && p.E > 0 && p.top > 0 && p.top <= p.E && p.E <= 4096 && p.ld % 64 == 0 && p.fp % 64 == 0, MYNN_ERR_INVALID,
                 "experts: top %d of %d, %d x %d", p.top, p.E, p.ld, p.fp);
    return 0;
}
int expert_gateup_row(const ExpertParams &p, int dtype, hipStream_t s) {
    int rc = check_experts(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.x && p.logits && p.hmid && p.chosen, MYNN_ERR_INVALID, "experts: null operand");
    const size_t lds = (size_t)(p.ld + p.E) * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        int rc2 = raise_lds(expert_gateup_row_kernel<T>, lds);
        if (rc2) return rc2;
        const int want = (p.fp / 2 + kRowW - 1) / kRowW, most = std::max(1, 1024 / p.top);
        MYNN_LAUNCH(expert_gateup_row_kernel<T>, dim3(std::min(want, most), p.top), dim3(kRowT), lds, s, p);
        return launch_status("expert_gateup_row_kernel");
    });
}
int expert_down_row(const ExpertParams &p, int dtype, hipStream_t s) {
    int rc = check_experts(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.hmid && p.chosen && p.y, MYNN_ERR_INVALID, "experts: null operand");
    const size_t lds = (size_t)p.top * p.fp * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        int rc2 = raise_lds(expert_down_row_kernel<T>, lds);
        if (rc2) return rc2;
        MYNN_LAUNCH(expert_down_row_kernel<T>, dim3(std::min((p.ld / 2 + kRowW - 1) / kRowW, 1024)), dim3(kRowT), lds, s, p);
        return launch_status("expert_down_row_kernel");
    });
}

// ---- several rows -------------------------------------------------------------------------------------------------------
// NR rows per workgroup: the rows in LDS, a wave per expert in turn
constexpr int kRouteRows = 8;
template <typename T>
__global__ __launch_bounds__(kRowT) void route_rows_kernel(ExpertParams p, int nr) {
    extern __shared__ __align__(16) float sm[];  // [nr][ld], [nr][E]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, row0 = blockIdx.x * nr, n = min(nr, p.rows - row0);
    float *z = sm + (size_t)nr * p.ld;
    for (int k = tid * 4; k < n * p.ld; k += kRowT * 4) *(float4 *)(sm + k) = *(const float4 *)(p.x + (size_t)row0 * p.ld + k);
    __syncthreads();
    for (int e = wave; e < p.E; e += kRowW) {
        const T *w = (const T *)p.router + (size_t)e * p.ld;
        float acc[kRouteRows] = {};
        for (int c = lane * 8; c < p.ld; c += 512) {
            float f[8];
            load8<T>(w + c, f);
#pragma unroll
            for (int i = 0; i < kRouteRows; i++)
                if (i < n) {
                    const float4 a = *(const float4 *)(sm + (size_t)i * p.ld + c), b = *(const float4 *)(sm + (size_t)i * p.ld + c + 4);
                    acc[i] = fmaf(f[0], a.x, fmaf(f[1], a.y, fmaf(f[2], a.z, fmaf(f[3], a.w, acc[i]))));
                    acc[i] = fmaf(f[4], b.x, fmaf(f[5], b.y, fmaf(f[6], b.z, fmaf(f[7], b.w, acc[i]))));
                }
        }
#pragma unroll
        for (int i = 0; i < kRouteRows; i++) {
            acc[i] = wave_sum(acc[i]);
            if (lane == 0 && i < n) z[i * p.E + e] = acc[i];
        }
    }
    __syncthreads();
    for (int i = wave; i < n; i += kRowW)
        for (int x = 0; x < p.top; x++) {
            const int e = take_largest(z + i * p.E, p.E, 0);
            const float v = z[i * p.E + e];
            __builtin_amdgcn_wave_barrier();
            if (lane == 0) {
                p.choice[(size_t)(row0 + i) * p.top + x] = e;
                p.score[(size_t)(row0 + i) * p.top + x] = sigmoidf(v);
                z[i * p.E + e] = -INFINITY;
            }
            __builtin_amdgcn_s_waitcnt(0xC07F);
            __builtin_amdgcn_wave_barrier();
        }
}
int expert_route(const ExpertParams &p, int dtype, hipStream_t s) {
    int rc = check_experts(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.x && p.router && p.choice && p.score && p.rows > 0, MYNN_ERR_INVALID, "experts: null operand");
    const int nr = std::max(1, std::min<int>(kRouteRows, (int)(kExpertLds / ((size_t)(p.ld + p.E) * 4))));
    const size_t lds = (size_t)nr * (p.ld + p.E) * 4;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        int rc2 = raise_lds(route_rows_kernel<T>, lds);
        if (rc2) return rc2;
        MYNN_LAUNCH(route_rows_kernel<T>, dim3((p.rows + nr - 1) / nr), dim3(kRowT), lds, s, p, nr);
        return launch_status("route_rows_kernel");
    });
}

// One workgroup: counts per expert, whole tiles per expert, then every assignment takes a place of its expert's.
constexpr int kSortT = 1024;
__global__ __launch_bounds__(kSortT) void sort_kernel(const int32_t *choice, int n, int E, int group_rows, int max_tiles, int32_t *tile_expert, int32_t *slot) {
    extern __shared__ int32_t cnt[];  // [E] counts, then next places
    const int tid = threadIdx.x;
    for (int e = tid; e < E; e += kSortT) cnt[e] = 0;
    for (int i = tid; i < max_tiles; i += kSortT) tile_expert[i] = -1;
    for (int i = tid; i < max_tiles * group_rows; i += kSortT) slot[i] = -1;
    __syncthreads();
    for (int i = tid; i < n; i += kSortT) atomicAdd(&cnt[choice[i]], 1);
    __syncthreads();
    if (tid == 0) {
        int tile = 0;
        for (int e = 0; e < E; e++) {
            const int first = tile, tiles = (cnt[e] + group_rows - 1) / group_rows;
            for (int t = 0; t < tiles; t++) tile_expert[tile++] = e;
            cnt[e] = first * group_rows;
        }
    }
    __syncthreads();
    for (int i = tid; i < n; i += kSortT) slot[atomicAdd(&cnt[choice[i]], 1)] = i;
}
int expert_sort(const ExpertParams &p, hipStream_t s) {
    MYNN_REQUIRE(p.choice && p.tile_expert && p.slot && p.rows > 0, MYNN_ERR_INVALID, "experts: null operand");
    const int gr = expert_group_rows(p.rows, p.E, p.top);
    MYNN_LAUNCH(sort_kernel, dim3(1), dim3(kSortT), (size_t)p.E * 4, s, p.choice, p.rows * p.top, p.E, gr, expert_tiles(p.rows, p.E, p.top, gr), p.tile_expert, p.slot);
    return launch_status("sort_kernel");
}

int expert_gateup(const ExpertParams &p, int dtype, hipStream_t s) {
    int rc = check_experts(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.act && p.hsort && p.score && p.slot && p.tile_expert, MYNN_ERR_INVALID, "experts: null operand");
    const int gr = expert_group_rows(p.rows, p.E, p.top);
    GroupedRows g{p.tile_expert, p.slot, p.score, p.top, true, expert_tiles(p.rows, p.E, p.top, gr), gr, (size_t)2 * p.fp * p.ld};
    return gemm_grouped(p.hsort, p.act, p.gu, g, 2 * p.fp, p.ld, GEMM_SILU, dtype, s);
}
int expert_down(const ExpertParams &p, int dtype, hipStream_t s) {
    int rc = check_experts(p);
    if (rc) return rc;
    MYNN_REQUIRE(p.hsort && p.y && p.slot && p.tile_expert && (p.top == 1 || p.parts), MYNN_ERR_INVALID, "experts: null operand");
    const int gr = expert_group_rows(p.rows, p.E, p.top);
    GroupedRows g{p.tile_expert, p.slot, nullptr, p.top, false, expert_tiles(p.rows, p.E, p.top, gr), gr, (size_t)p.ld * p.fp};
    return gemm_grouped(p.top == 1 ? p.y : (void *)p.parts, p.hsort, p.down, g, p.ld, p.fp, p.top == 1 ? GEMM_PLAIN : GEMM_F32, dtype, s);
}

template <typename T> __global__ __launch_bounds__(256) void expert_sum_kernel(T *y, const float *parts, int top, int ld, size_t total) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= total) return;
    const size_t row = i / ld, c = i % ld;
    float4 a = float4{0.f, 0.f, 0.f, 0.f};
    for (int x = 0; x < top; x++) {
        const float4 v = *(const float4 *)(parts + (row * top + x) * ld + c);
        a.x += v.x; a.y += v.y; a.z += v.z; a.w += v.w;
    }
    store4<T>(y + i, a);
}
int expert_sum(const ExpertParams &p, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.y && p.parts && p.rows > 0, MYNN_ERR_INVALID, "experts: null operand");
    const size_t total = (size_t)p.rows * p.ld;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(expert_sum_kernel<T>, dim3((unsigned)((total / 4 + 255) / 256)), dim3(256), 0, s, (T *)p.y, p.parts, p.top, p.ld, total);
        return launch_status("expert_sum_kernel");
    });
}

}  // namespace mynn
