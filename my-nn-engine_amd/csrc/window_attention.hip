// Window attention with kept first tokens (see window_attention.h).  Two kernels over the same cache rows [keys | values]:
//   window_rows_kernel: 16-byte pieces of a key across a group of lanes, several keys per wave at a time, up to four query
//     heads of a key/value head per workgroup; ranges of the visible keys per workgroup, merged by window_merge_kernel.
//     Decode, f32 throughout, and every head size.
//   window_prefill_kernel: flash attention on the matrix cores for prompts.  A workgroup of query rows walks the tiles that
//     hold kept tokens, then the tiles its rows' windows reach.
#include <algorithm>
#include <type_traits>

#include "dense_load.h"
#include "window_attention.h"

namespace mynn {

// The keys position `pos` sees, in rising order: index n < sinks is key n, the rest follow from `lo`.
struct Visible {
    int sinks, lo, count;
    __device__ int key(int n) const { return n < sinks ? n : lo + n - sinks; }
};
__device__ inline Visible visible_keys(int pos, int window, int keep_first) {
    const int first = window > 0 ? max(0, pos - window + 1) : 0;
    Visible v;
    v.sinks = min(keep_first, first);
    v.lo = first;
    v.count = v.sinks + pos + 1 - first;
    return v;
}
// length of a range when `count` keys are cut into at most nsplit
constexpr int kMinKeys = 64;
__device__ inline int range_keys(int count, int nsplit) { return max(kMinKeys, ((count + nsplit - 1) / nsplit + 15) / 16 * 16); }

constexpr int kRowsThreads = 256, kRowsWaves = 4;

// LPK lanes per key (8 values each), RH query heads of one kv head.
template <typename T, int LPK, int RH>
__global__ __launch_bounds__(kRowsThreads) void window_rows_kernel(WindowAttnParams p) {
    constexpr int KPW = 64 / LPK, UN = 4;  // keys of a wave at a time, and how many such groups are requested together
    __shared__ float s_ml[kRowsWaves][RH][2];
    extern __shared__ __align__(16) float s_o[];  // [kRowsWaves][RH][LPK * 8]
    const ParallelDims &d = p.d;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, part = lane % LPK, slot = lane / LPK;
    const int per_kv = d.H / d.G, chunks = (per_kv + RH - 1) / RH;
    const int g = blockIdx.x / chunks, h0 = g * per_kv + (blockIdx.x % chunks) * RH, nh = min(RH, (g + 1) * per_kv - h0);
    const int row = blockIdx.z, b = row / p.S, split = blockIdx.y;
    const int pos = *p.d_past + row % p.S;
    const Visible vis = visible_keys(pos, p.window, p.keep_first);
    const int range = range_keys(vis.count, p.nsplit), n0 = split * range, n1 = min(vis.count, n0 + range);
    const bool have = part * 8 < d.dimp;
    float q[RH][8], acc[RH][8], m[RH], l[RH];
#pragma unroll
    for (int i = 0; i < RH; i++) {
        m[i] = -INFINITY;
        l[i] = 0.f;
#pragma unroll
        for (int e = 0; e < 8; e++) q[i][e] = acc[i][e] = 0.f;
        if (have && i < nh) {
            load8<T>((const T *)p.q + (size_t)row * d.qcols() + (h0 + i) * d.dimp + part * 8, q[i]);
#pragma unroll
            for (int e = 0; e < 8; e++) q[i][e] *= p.scale;
        }
    }
    const T *cache = (const T *)p.cache + g * d.dimp + min(part * 8, d.dimp - 8);
    const int vofs = d.G * d.dimp;
    for (int n = n0 + wave * KPW * UN; n < n1; n += kRowsWaves * KPW * UN) {
        Row8<T> kr[UN], vr[UN];
#pragma unroll
        for (int u = 0; u < UN; u++) {
            const T *at = cache + window_cache_row(p, b, vis.key(min(n + u * KPW + slot, n1 - 1))) * d.row();
            kr[u].get(at);
            vr[u].get(at + vofs);
        }
#pragma unroll
        for (int u = 0; u < UN; u++) {
            float kf[8], vf[8], sc[RH];
            kr[u].widen(kf);
            vr[u].widen(vf);
            const bool live = n + u * KPW + slot < n1;
#pragma unroll
            for (int i = 0; i < RH; i++) {
                float a = 0.f;
#pragma unroll
                for (int e = 0; e < 8; e++) a = fmaf(q[i][e], kf[e], a);
                sc[i] = group_sum<LPK>(a);
            }
#pragma unroll
            for (int i = 0; i < RH; i++) {
                if (!live) continue;
                const float mn = fmaxf(m[i], sc[i]), f = expf(m[i] - mn), pe = expf(sc[i] - mn);
                m[i] = mn;
                l[i] = fmaf(l[i], f, pe);
#pragma unroll
                for (int e = 0; e < 8; e++) acc[i][e] = fmaf(pe, vf[e], acc[i][e] * f);
            }
        }
    }
    // merge the key slots of the wave, then the waves
#pragma unroll
    for (int i = 0; i < RH; i++) {
#pragma unroll
        for (int off = LPK; off < 64; off <<= 1) {
            const float om = __shfl_xor(m[i], off, 64), ol = __shfl_xor(l[i], off, 64);
            const float mn = fmaxf(m[i], om);
            const float fa = m[i] > -INFINITY ? expf(m[i] - mn) : 0.f, fb = om > -INFINITY ? expf(om - mn) : 0.f;
            l[i] = l[i] * fa + ol * fb;
#pragma unroll
            for (int e = 0; e < 8; e++) acc[i][e] = acc[i][e] * fa + __shfl_xor(acc[i][e], off, 64) * fb;
            m[i] = mn;
        }
        if (slot == 0) {
#pragma unroll
            for (int e = 0; e < 8; e++) s_o[(wave * RH + i) * LPK * 8 + part * 8 + e] = acc[i][e];
            if (part == 0) {
                s_ml[wave][i][0] = m[i];
                s_ml[wave][i][1] = l[i];
            }
        }
    }
    __syncthreads();
    for (int idx = tid; idx < nh * d.dimp; idx += kRowsThreads) {
        const int i = idx / d.dimp, c = idx % d.dimp;
        float mm = -INFINITY, ll = 0.f, o = 0.f;
#pragma unroll
        for (int w = 0; w < kRowsWaves; w++) mm = fmaxf(mm, s_ml[w][i][0]);
#pragma unroll
        for (int w = 0; w < kRowsWaves; w++)
            if (s_ml[w][i][0] > -INFINITY) {
                const float f = expf(s_ml[w][i][0] - mm);
                ll = fmaf(s_ml[w][i][1], f, ll);
                o = fmaf(s_o[(w * RH + i) * LPK * 8 + c], f, o);
            }
        if (p.nsplit == 1) Elem<T>::st((T *)p.out, (size_t)row * d.acols() + (h0 + i) * d.dimp + c, o / ll * p.out_scale);
        else {
            const size_t at = ((size_t)row * d.H + h0 + i) * p.nsplit + split;
            p.part_o[at * d.dimp + c] = o;
            if (c == 0) {
                p.part_ml[at * 2] = mm;
                p.part_ml[at * 2 + 1] = ll;
            }
        }
    }
}

template <typename T> __global__ __launch_bounds__(64) void window_merge_kernel(WindowAttnParams p) {
    const ParallelDims &d = p.d;
    const int h = blockIdx.x, row = blockIdx.y, lane = threadIdx.x;
    const size_t at = ((size_t)row * d.H + h) * p.nsplit;
    const int count = visible_keys(*p.d_past + row % p.S, p.window, p.keep_first).count, range = range_keys(count, p.nsplit);
    const int live = (count + range - 1) / range;  // (at most 64: one range per lane)
    const float m = lane < live ? p.part_ml[(at + lane) * 2] : -INFINITY, l = lane < live ? p.part_ml[(at + lane) * 2 + 1] : 0.f;
    const float mm = wave_max(m), f = lane < live ? expf(m - mm) : 0.f, ll = wave_sum(l * f);
    const float w = f / ll * p.out_scale;
    for (int c0 = 0; c0 < d.dimp; c0 += 64) {
        const int c = min(c0 + lane, d.dimp - 1);
        float o = 0.f;
        for (int r = 0; r < live; r += 8) {  // (lanes past the last range weigh nothing)
            float v[8];
#pragma unroll
            for (int u = 0; u < 8; u++) v[u] = p.part_o[(at + min(r + u, live - 1)) * d.dimp + c];
#pragma unroll
            for (int u = 0; u < 8; u++) o = fmaf(__shfl(w, r + u, 64), v[u], o);
        }
        if (c0 + lane < d.dimp) Elem<T>::st((T *)p.out, (size_t)row * d.acols() + h * d.dimp + c, o);
    }
}

bool window_attention_dim_supported(int dimp) { return dimp <= 512; }

static int rows_heads(const ParallelDims &d) {
    const int r = d.H / d.G;
    return r >= 4 ? 4 : r >= 2 ? 2 : 1;
}
int window_attention_splits(int B, int S, const ParallelDims &d, int window, int keep_first, int max_seq) {
    const long most = window > 0 ? std::min<long>(max_seq, (long)window + keep_first) : max_seq;
    const int rh = rows_heads(d);
    const long groups = (long)d.G * ((d.H / d.G + rh - 1) / rh) * B * S;
    return (int)std::max(1L, std::min({512 / groups, (most + kMinKeys - 1) / kMinKeys, 64L}));
}

static int check_window(const WindowAttnParams &p) {
    MYNN_REQUIRE(p.q && p.cache && p.out && p.d_past && (p.nsplit == 1 || (p.part_o && p.part_ml)), MYNN_ERR_INVALID, "window attention: null operand");
    MYNN_REQUIRE(p.nsplit >= 1 && p.nsplit <= 64 && window_attention_dim_supported(p.d.dimp) && (long)p.B * p.S <= 65535, MYNN_ERR_UNSUPPORTED,
                 "window attention: %d ranges, heads of %d, %d rows", p.nsplit, p.d.dim, p.B * p.S);
    return 0;
}

int window_attention_rows(const WindowAttnParams &p, int dtype, hipStream_t s) {
    int rc = check_window(p);
    if (rc) return rc;
    const ParallelDims &d = p.d;
    const int rh = rows_heads(d);
    const dim3 grid(d.G * ((d.H / d.G + rh - 1) / rh), p.nsplit, p.B * p.S);
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        auto go = [&](auto lpk, auto nh) {
            constexpr int LPK = decltype(lpk)::value, RH = decltype(nh)::value;
            MYNN_LAUNCH((window_rows_kernel<T, LPK, RH>), grid, dim3(kRowsThreads), (size_t)kRowsWaves * RH * LPK * 8 * 4, s, p);
            return launch_status("window_rows_kernel");
        };
        auto heads = [&](auto lpk) {
            if (rh == 4) return go(lpk, std::integral_constant<int, 4>{});
            if (rh == 2) return go(lpk, std::integral_constant<int, 2>{});
            return go(lpk, std::integral_constant<int, 1>{});
        };
        if (d.dimp <= 64) return heads(std::integral_constant<int, 8>{});
        if (d.dimp <= 128) return heads(std::integral_constant<int, 16>{});
        if (d.dimp <= 256) return heads(std::integral_constant<int, 32>{});
        return heads(std::integral_constant<int, 64>{});
    });
}
int window_attention_merge(const WindowAttnParams &p, int dtype, hipStream_t s) {
    int rc = check_window(p);
    if (rc) return rc;
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        MYNN_LAUNCH(window_merge_kernel<T>, dim3(p.d.H, p.B * p.S), dim3(64), 0, s, p);
        return launch_status("window_merge_kernel");
    });
}

// ---- prompts ------------------------------------------------------------------------------------------------------------
// WAVES waves of 32 query rows of one head, 64-key tiles, head size up to D.  Per tile: S^T = K . Q^T (K from LDS, Q in
// registers), softmax with one query per lane, O^T += V^T . P^T with P in the registers the first product left it in.
template <typename T, int D, int WAVES>
__global__ __launch_bounds__(64 * WAVES, 2) void window_prefill_kernel(WindowAttnParams p, int past) {
    constexpr int NT = 64 * WAVES, KEYS = 64, LDK = D + 8, LDV = KEYS + 4, KSTEPS = D / 16, DT = D / 32;
    constexpr int CHK = KEYS * D / 8 / NT, CHV = CHK;
    static_assert(KEYS * D / 8 % NT == 0 && (CHV == 2 || CHV == 4), "whole pieces per thread");
    extern __shared__ __align__(16) uint16_t wp_smem[];
    uint16_t *Ks = wp_smem, *Vt = wp_smem + 2 * KEYS * LDK;
    const ParallelDims &d = p.d;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, g = lane >> 5;
    const int h = blockIdx.x, kvh = h / (d.H / d.G), b = blockIdx.z, S = p.S, window = p.window, keep = p.keep_first;
    const int q_blk = ((int)gridDim.y - 1 - (int)blockIdx.y) * 32 * WAVES;
    const int qrow = q_blk + wave * 32 + col, qrow_c = min(qrow, S - 1), my_pos = past + qrow_c;
    const int my_first = window > 0 ? my_pos - window + 1 : 0;
    const int wave_lo = past + min(q_blk + wave * 32, S - 1), wave_hi = past + min(q_blk + wave * 32 + 31, S - 1);  // positions of the wave's rows
    const int wave_first = window > 0 ? max(0, wave_lo - window + 1) : 0;        // first key any row of the wave sees in its window
    const int wave_all = window > 0 ? max(0, wave_hi - window + 1) : 0;          // first key every row sees
    const int blk_bound = past + min(q_blk + 32 * WAVES - 1, S - 1) + 1;
    const int blk_first = window > 0 ? max(0, past + q_blk - window + 1) : 0;
    const int t_win = blk_first / KEYS, t_sink = min((keep + KEYS - 1) / KEYS, t_win);  // tiles of kept tokens ahead of the window's
    const int ntiles = t_sink + (blk_bound + KEYS - 1) / KEYS - t_win;
    auto tile_at = [&](int n) { return n < t_sink ? n : n - t_sink + t_win; };
    const int32_t *table = p.paging.table ? p.paging.table + (size_t)b * p.paging.pages_per_seq : nullptr;
    const int psh = p.paging.shift, pmask = (1 << psh) - 1;
    // (a tile starts at a multiple of 64 and a page holds a multiple of 64 rows: a tile lies in one page)
    auto page_of = [&](int n) { return table ? table[tile_at(min(n, ntiles - 1)) * KEYS >> psh] : 0; };

    const int key0 = (tid / (D / 8)) * CHV, dd = (tid % (D / 8)) * 8;  // thread -> CHV neighbouring keys, 8 dimensions of them
    const T *base = (const T *)p.cache + kvh * d.dimp;
    U4 rk[CHK], rv[CHV];
    auto load_tile = [&](int n, int page) {
        const int t0 = tile_at(n) * KEYS;
#pragma unroll
        for (int i = 0; i < CHV; i++) {
            const int key = min(t0 + key0 + i, blk_bound - 1);
            const size_t row = table ? ((size_t)page << psh) + (key & pmask) : (size_t)b * p.max_seq + key;
            rk[i] = rv[i] = U4{0u, 0u, 0u, 0u};
            if (dd < d.dimp) {
                rk[i] = *(const U4 *)(base + row * d.row() + dd);
                rv[i] = *(const U4 *)(base + row * d.row() + d.G * d.dimp + dd);
            }
        }
    };
    auto store_tile = [&](int buf) {
#pragma unroll
        for (int i = 0; i < CHK; i++) *(U4 *)&Ks[buf * KEYS * LDK + (key0 + i) * LDK + dd] = rk[i];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            uint32_t w[CHV];
#pragma unroll
            for (int c = 0; c < CHV; c++) w[c] = i == 0 ? rv[c].x : i == 1 ? rv[c].y : i == 2 ? rv[c].z : rv[c].w;
            uint16_t *lo = &Vt[buf * D * LDV + (dd + 2 * i) * LDV + key0], *hi = lo + LDV;
            if constexpr (CHV == 2) {
                *(uint32_t *)lo = __builtin_amdgcn_perm(w[1], w[0], 0x05040100u);
                *(uint32_t *)hi = __builtin_amdgcn_perm(w[1], w[0], 0x07060302u);
            } else {
                *(uint2 *)lo = uint2{__builtin_amdgcn_perm(w[1], w[0], 0x05040100u), __builtin_amdgcn_perm(w[3], w[2], 0x05040100u)};
                *(uint2 *)hi = uint2{__builtin_amdgcn_perm(w[1], w[0], 0x07060302u), __builtin_amdgcn_perm(w[3], w[2], 0x07060302u)};
            }
        }
    };

    load_tile(0, page_of(0));
    const size_t prow = (size_t)b * S + qrow_c;
    const T *Q = (const T *)p.q + prow * d.qcols() + h * d.dimp;
    U4 qf[KSTEPS];
#pragma unroll
    for (int ks = 0; ks < KSTEPS; ks++) {
        qf[ks] = U4{0u, 0u, 0u, 0u};
        if (16 * ks < d.dimp) qf[ks] = *(const U4 *)(Q + 16 * ks + 8 * g);
    }
    f16x_t o[DT];
#pragma unroll
    for (int t = 0; t < DT; t++)
#pragma unroll
        for (int e = 0; e < 16; e++) o[t][e] = 0.f;
    float m = -INFINITY, l = 0.f;  // running maximum in units of log2
    const float scale2 = p.scale * 1.4426950408889634f;

    auto tile = [&](int buf, int k0, auto masked) {
        constexpr bool MASKED = decltype(masked)::value;
        const uint16_t *Kb = Ks + buf * KEYS * LDK, *Vb = Vt + buf * D * LDV;
        f16x_t s[2];
#pragma unroll
        for (int hf = 0; hf < 2; hf++)
#pragma unroll
            for (int e = 0; e < 16; e++) s[hf][e] = 0.f;
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ks++)
#pragma unroll
            for (int hf = 0; hf < 2; hf++)
                s[hf] = Mfma<T>::run(*(const U4 *)&Kb[(32 * hf + col) * LDK + 16 * ks + 8 * g], qf[ks], s[hf]);
        float mloc = -INFINITY;
#pragma unroll
        for (int hf = 0; hf < 2; hf++)
#pragma unroll
            for (int e = 0; e < 16; e++) {
                s[hf][e] *= scale2;
                if (MASKED) {
                    const int key = k0 + 32 * hf + 8 * (e >> 2) + 4 * g + (e & 3);
                    if (key > my_pos || (key < my_first && key >= keep)) s[hf][e] = -INFINITY;
                }
                mloc = fmaxf(mloc, s[hf][e]);
            }
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
        const float mn = fmaxf(m, mloc);
        float corr = 1.f;
        if (MASKED && mn == -INFINITY) {
#pragma unroll
            for (int hf = 0; hf < 2; hf++)
#pragma unroll
                for (int e = 0; e < 16; e++) s[hf][e] = 0.f;
        } else {
            corr = __builtin_amdgcn_exp2f(m - mn);
            float ls = 0.f;
#pragma unroll
            for (int hf = 0; hf < 2; hf++)
#pragma unroll
                for (int e = 0; e < 16; e++) {
                    s[hf][e] = __builtin_amdgcn_exp2f(s[hf][e] - mn);
                    ls += s[hf][e];
                }
            l = fmaf(l, corr, ls);
            m = mn;
        }
        if (__builtin_amdgcn_ballot_w64(corr != 1.f) != 0) {
#pragma unroll
            for (int t2 = 0; t2 < DT; t2++)
#pragma unroll
                for (int e = 0; e < 16; e++) o[t2][e] *= corr;
        }
#pragma unroll
        for (int st = 0; st < 4; st++) {
            const f16x_t &ph = s[st >> 1];
            const int e0 = 8 * (st & 1);
            const U4 pf = U4{pack2<T>(ph[e0 + 0], ph[e0 + 1]), pack2<T>(ph[e0 + 2], ph[e0 + 3]),
                             pack2<T>(ph[e0 + 4], ph[e0 + 5]), pack2<T>(ph[e0 + 6], ph[e0 + 7])};
#pragma unroll
            for (int t2 = 0; t2 < DT; t2++) {
                const uint16_t *vr = &Vb[(32 * t2 + col) * LDV + 16 * st + 4 * g];
                const uint2 lo = *(const uint2 *)vr, hi = *(const uint2 *)(vr + 8);
                o[t2] = Mfma<T>::run(U4{lo.x, lo.y, hi.x, hi.y}, pf, o[t2]);
            }
        }
    };

    store_tile(0);
    load_tile(min(1, ntiles - 1), page_of(1));
    int page_next = page_of(2);
    __syncthreads();
    for (int n = 0; n < ntiles; n++) {
        // tile n is in LDS, tile n + 1 in registers; its buffer was released by the last barrier
        if (n + 1 < ntiles) store_tile((n + 1) & 1);
        load_tile(min(n + 2, ntiles - 1), page_next);
        page_next = page_of(n + 3);
        const int k0 = tile_at(n) * KEYS;
        if (k0 >= wave_all && k0 + KEYS <= wave_lo + 1) tile(n & 1, k0, std::false_type{});
        else if (k0 <= wave_hi && (k0 + KEYS > wave_first || k0 < keep)) tile(n & 1, k0, std::true_type{});
        __syncthreads();
    }

    l += __shfl_xor(l, 32, 64);
    if (qrow < S) {
        T *out = (T *)p.out + prow * d.acols() + h * d.dimp;
        const float f = p.out_scale / l;
#pragma unroll
        for (int t2 = 0; t2 < DT; t2++)
#pragma unroll
            for (int e4 = 0; e4 < 4; e4++) {
                const int c = 32 * t2 + 8 * e4 + 4 * g;
                if (c < d.dimp) *(uint2 *)(out + c) = uint2{pack2<T>(o[t2][4 * e4 + 0] * f, o[t2][4 * e4 + 1] * f), pack2<T>(o[t2][4 * e4 + 2] * f, o[t2][4 * e4 + 3] * f)};
            }
    }
}

bool window_prefill_supported(const ParallelDims &d, int dtype) { return dtype == MYNN_BF16 && d.dimp <= 128; }

int window_attention_prefill(const WindowAttnParams &p, int past, int dtype, hipStream_t s) {
    int rc = check_window(p);
    if (rc) return rc;
    MYNN_REQUIRE(window_prefill_supported(p.d, dtype) && past >= 0 && past + p.S <= p.max_seq && p.B <= 65535, MYNN_ERR_INVALID,
                 "window prefill attention: rows %d + %d of %d", past, p.S, p.max_seq);
    MYNN_REQUIRE(!p.paging.table || (1 << p.paging.shift) >= 64, MYNN_ERR_UNSUPPORTED, "window prefill attention: pages of %d rows", 1 << p.paging.shift);
    auto go = [&](auto kernel, int D) {
        constexpr int waves = 4;
        const size_t lds = ((size_t)2 * 64 * (D + 8) + (size_t)2 * D * 68) * 2;
        if (lds > 60 * 1024) MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        MYNN_LAUNCH(kernel, dim3(p.d.H, (p.S + 32 * waves - 1) / (32 * waves), p.B), dim3(64 * waves), lds, s, p, past);
        return launch_status("window_prefill_kernel");
    };
    if (p.d.dimp <= 64) return go(window_prefill_kernel<bf16_t, 64, 4>, 64);
    return go(window_prefill_kernel<bf16_t, 128, 4>, 128);
}

}  // namespace mynn
