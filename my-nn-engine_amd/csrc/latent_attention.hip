// Latent attention: keys and values of all heads are linear images of one normed latent per token, which (with one rotated
// key part shared by the heads) is all the cache holds.
//
// Two forms of the same product, chosen by the number of query rows:
//   absorbed (decode, short portions): score_h(j) = (W_uk[h]^T q_h) . c_j + q_rot . k_rot_j and
//     out_h = W_uv[h] (sum_j p_j c_j), so all heads attend to the SAME cache rows: one read of the cache serves every head.
//     latent_prepare_kernel makes the taken-in queries, latent_absorbed_kernel walks a key range with 16 or 32 (query,
//     head) rows per workgroup on the matrix cores, latent_out_kernel merges the ranges and applies W_uv and the gate.
//   expanded (prompts): K = W_uk c, V = W_uv c for every visible token by one GEMM, then flash attention over query / key
//     width dim + rot_dim and value width vdim (latent_prefill_kernel), the gate in the store.
// latent_absorbed_plain_kernel is the absorbed product for f32 and for shapes the matrix-core kernel has no form for.
#include <algorithm>
#include <type_traits>

#include "dense_load.h"
#include "latent_attention.h"

namespace mynn {

typedef float lf4_t __attribute__((ext_vector_type(4)));
template <typename T> struct MfmaL16;
template <> struct MfmaL16<bf16_t> {
    __device__ static lf4_t run(const U4 &a, const U4 &b, lf4_t c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(b8_t, a), __builtin_bit_cast(b8_t, b), c, 0, 0, 0);
    }
};

__device__ inline size_t latent_row(const LatentParams &p, int b, int r) { return kv_cache_row(p.paging, b, 0, r, 1, p.max_seq); }

// pair i of a rotated part at position pos
__device__ inline void rotate_pair(const LatentParams &p, int pos, int i, float &u, float &v) {
    if (2 * i >= p.rot_dims) return;  // (dimensions past the rotated ones pass)
    const float2 cs = p.rot[(size_t)pos * (p.rot_dims / 2) + i];
    const float a = u * cs.x - v * cs.y, b = v * cs.x + u * cs.y;
    u = a;
    v = b;
}

// ---- prepare: workgroup x == 0 of a row makes the cache row, the others the queries ---------------------------------
constexpr int kPrepThreads = 256, kPrepCols = 128;
template <typename T, bool ABSORB>
__global__ __launch_bounds__(kPrepThreads) void latent_prepare_kernel(LatentParams p) {
    __shared__ float sm[kPrepThreads * 8 + 8];
    const LatentDims &d = p.d;
    const int row = blockIdx.y, b = row / p.S, pos = *p.d_past + row % p.S, tid = threadIdx.x;
    T *proj = (T *)p.proj + (size_t)row * d.n_in();
    if (blockIdx.x == 0) {
        const T *lat = proj + d.qcols(), *kr = lat + d.rp;
        T *dst = (T *)p.cache + latent_row(p, b, pos) * d.lw();
        // (one sequence, expanded form: the row also goes where the expansion reads it)
        T *c2 = !ABSORB && p.B == 1 ? (T *)p.c_rows + (size_t)pos * d.rp : nullptr, *r2 = c2 ? (T *)p.rot_rows + (size_t)pos * d.rotp : nullptr;
        float ss = 0.f;
        for (int k = tid; k < d.rank; k += kPrepThreads) {
            const float v = Elem<T>::ld(lat, k);
            ss += v * v;
        }
        ss = wave_sum(ss);
        if ((tid & 63) == 0) sm[tid >> 6] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf((sm[0] + sm[1] + sm[2] + sm[3]) / (float)d.rank + p.eps);
        for (int k = tid; k < d.rp; k += kPrepThreads) {
            const float v = k < d.rank ? Elem<T>::ld(lat, k) * inv * Elem<T>::ld((const T *)p.norm_w, k) : 0.f;
            Elem<T>::st(dst, k, v);
            if (c2) Elem<T>::st(c2, k, v);
        }
        for (int i = tid; i < d.rotp / 2; i += kPrepThreads) {
            float u = Elem<T>::ld(kr, 2 * i), v = Elem<T>::ld(kr, 2 * i + 1);
            rotate_pair(p, pos, i, u, v);
            Elem<T>::st(dst, d.rp + 2 * i, u);
            Elem<T>::st(dst, d.rp + 2 * i + 1, v);
            if (r2) {
                Elem<T>::st(r2, 2 * i, u);
                Elem<T>::st(r2, 2 * i + 1, v);
            }
        }
        return;
    }
    if constexpr (!ABSORB) {
        const int half = p.rot_dims / 2;
        for (int j = tid; j < d.H * half; j += kPrepThreads) {
            T *q = proj + (j / half) * d.dk() + d.dimp;
            const int i = j % half;
            float u = Elem<T>::ld(q, 2 * i), v = Elem<T>::ld(q, 2 * i + 1);
            rotate_pair(p, pos, i, u, v);
            Elem<T>::st(q, 2 * i, u);
            Elem<T>::st(q, 2 * i + 1, v);
        }
    } else {
        const int nchunk = (d.rp + kPrepCols - 1) / kPrepCols;
        const int h = ((int)blockIdx.x - 1) / nchunk, chunk = ((int)blockIdx.x - 1) % nchunk;
        const int c0 = chunk * kPrepCols, cols = min(kPrepCols, d.rp - c0);
        const T *q = proj + h * d.dk();
        T *dst = (T *)p.q_abs + ((size_t)row * d.H + h) * d.lw();
        // thread = (column group of 8, every ndg-th of the head's dimensions); the groups' sums meet in LDS
        const int ncg = cols >> 3, ndg = kPrepThreads / ncg, cg = tid % ncg, dg = tid / ncg;
        float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (dg < ndg) {
            const T *w = (const T *)p.ukv + (size_t)h * d.dimp * d.rp + c0 + cg * 8;
#pragma unroll 8
            for (int k = dg; k < d.dim; k += ndg) {
                float f[8];
                load8<T>(w + (size_t)k * d.rp, f);
                const float qv = Elem<T>::ld(q, k);
#pragma unroll
                for (int e = 0; e < 8; e++) acc[e] = fmaf(qv, f[e], acc[e]);
            }
#pragma unroll
            for (int e = 0; e < 8; e++) sm[dg * cols + cg * 8 + e] = acc[e];
        }
        __syncthreads();
        for (int c = tid; c < cols; c += kPrepThreads) {
            float t = 0.f;
            for (int g = 0; g < ndg; g++) t += sm[g * cols + c];
            Elem<T>::st(dst, c0 + c, t);
        }
        if (chunk == 0)
            for (int i = tid; i < d.rotp / 2; i += kPrepThreads) {
                float u = Elem<T>::ld(q, d.dimp + 2 * i), v = Elem<T>::ld(q, d.dimp + 2 * i + 1);
                rotate_pair(p, pos, i, u, v);
                Elem<T>::st(dst, d.rp + 2 * i, u);
                Elem<T>::st(dst, d.rp + 2 * i + 1, v);
            }
    }
}

int latent_prepare(const LatentParams &p, bool absorb, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.proj && p.norm_w && p.cache && p.rot && p.d_past && (!absorb || (p.ukv && p.q_abs)) && (absorb || p.B > 1 || (p.c_rows && p.rot_rows)), MYNN_ERR_INVALID, "latent prepare: null operand");
    MYNN_REQUIRE((long)p.B * p.S <= 65535, MYNN_ERR_UNSUPPORTED, "latent prepare: %d rows", p.B * p.S);
    const int nchunk = (p.d.rp + kPrepCols - 1) / kPrepCols;
    const dim3 grid(absorb ? 1 + p.d.H * nchunk : 2, p.B * p.S);
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        if (absorb) MYNN_LAUNCH((latent_prepare_kernel<T, true>), grid, dim3(kPrepThreads), 0, s, p);
        else MYNN_LAUNCH((latent_prepare_kernel<T, false>), grid, dim3(kPrepThreads), 0, s, p);
        return launch_status("latent_prepare_kernel");
    });
}

// ---- absorbed attention -------------------------------------------------------------------------------------------------
// Key ranges: the active rows are cut into at most nsplit ranges of a multiple of 64 rows.
constexpr int kTile = 64, kMinRange = 64;
__device__ __host__ inline int latent_range(int active, int nsplit) {
    const int r = ((active + nsplit - 1) / nsplit + kTile - 1) / kTile * kTile;
    return r < kMinRange ? kMinRange : r;
}

// One workgroup of eight waves: 16 * MT rows of a sequence's (query, head) pairs against one key range.  Tiles of 64 keys:
// the tile is staged in LDS (the next one waits in registers), the waves share the score product (by 16 keys and by query
// tile, or by halves of the row for MT == 1), every wave then takes the softmax of all rows and adds its own 32-column
// blocks of P . C.  CB: 32-column blocks per wave.  div: ceil(2^20 / (16-byte pieces of a row)).
constexpr int kAbsThreads = 512, kAbsWaves = kAbsThreads / 64;
template <typename T, int MT, int CB>
__global__ __launch_bounds__(kAbsThreads) void latent_absorbed_kernel(LatentParams p, unsigned div) {
    constexpr int KS = MT == 1 ? 2 : 1;                     // partial score products per (key, query)
    constexpr int NL = 4 * CB + 2, NQ = MT * (CB + 1);      // 16-byte pieces of a tile / of the queries per thread
    constexpr int SST = kTile + 4;
    static_assert(kTile == 64 && kAbsWaves == 8, "four key groups of 16, two score products each");
    extern __shared__ __align__(16) char smem[];
    const LatentDims &d = p.d;
    const int lw = d.lw(), ldc = lw + 8, cpr = lw >> 3;
    T *Cs = (T *)smem, *Qs = Cs + kTile * ldc;
    float *Ss = (float *)(Qs + 16 * MT * ldc);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, quad = lane >> 4;
    const int split = blockIdx.x, r0 = blockIdx.y * 16 * MT, b = blockIdx.z;
    const int nrows = p.S * d.H;
    // idx / cpr for idx < 8192, cpr <= 128 by a multiplication (idx * (div * cpr - 2^20) < 2^20)
    auto row_of = [&](int idx) { return (int)(((unsigned)idx * div) >> 20); };
    // the queries (rows past the end become zeros) are requested before anything waits for the context length
    U4 qv[NQ];
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const int idx = min(tid + i * kAbsThreads, 16 * MT * cpr - 1), r = row_of(idx);
        qv[i] = *(const U4 *)((const T *)p.q_abs + ((size_t)b * nrows + min(r0 + r, nrows - 1)) * lw + (idx - r * cpr) * 8);
    }
    const int past = *p.d_past;
    const int range = latent_range(past + p.S, p.nsplit);
    const int last_q = min(r0 + 16 * MT - 1, nrows - 1) / d.H;       // the furthest query of the workgroup
    const int k0 = split * range, k1 = min(min(past + p.S, k0 + range), past + last_q + 1);
    int bound[MT];  // keys the row of this lane's column sees
#pragma unroll
    for (int m = 0; m < MT; m++) bound[m] = min(past + min(r0 + 16 * m + col, nrows - 1) / d.H + 1, k1);

    float m_run[MT], l_run[MT];
    lf4_t acc[MT][CB][2];
#pragma unroll
    for (int m = 0; m < MT; m++) {
        m_run[m] = -INFINITY;
        l_run[m] = 0.f;
#pragma unroll
        for (int c = 0; c < CB; c++) acc[m][c][0] = acc[m][c][1] = lf4_t{0.f, 0.f, 0.f, 0.f};
    }

    const int psh = p.paging.shift, pmask = (1 << psh) - 1;
    const int32_t *table = p.paging.table ? p.paging.table + (size_t)b * p.paging.pages_per_seq : nullptr;
    const int ntiles = k1 > k0 ? (k1 - k0 + kTile - 1) / kTile : 0;
    // (a tile starts at a multiple of 64 and a page holds a multiple of 64 rows: a tile lies in one page, whose number
    // is asked for one tile ahead of the loads that need it)
    auto page_of = [&](int t) { return table ? table[(k0 + min(t, ntiles - 1) * kTile) >> psh] : 0; };
    U4 pre[NL];
    auto load_tile = [&](int t, int page) {
        const int t0 = k0 + t * kTile;
#pragma unroll
        for (int i = 0; i < NL; i++) {
            const int idx = min(tid + i * kAbsThreads, kTile * cpr - 1), r = row_of(idx);
            const int key = min(t0 + r, k1 - 1);
            const size_t row = table ? ((size_t)page << psh) + (key & pmask) : (size_t)b * p.max_seq + key;
            pre[i] = *(const U4 *)((const T *)p.cache + row * lw + (idx - r * cpr) * 8);
        }
    };
    int page_next = 0;
    if (ntiles) {
        load_tile(0, page_of(0));
        page_next = page_of(1);
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const int idx = tid + i * kAbsThreads, r = row_of(idx);
            if (idx < 16 * MT * cpr) *(U4 *)(Qs + r * ldc + (idx - r * cpr) * 8) = r0 + r < nrows ? qv[i] : U4{0u, 0u, 0u, 0u};
        }
    }
    const int nks = lw >> 5, nblk = d.rp >> 5;
    for (int t = 0; t < ntiles; t++) {
        __syncthreads();  // the tile before is no longer read
#pragma unroll
        for (int i = 0; i < NL; i++) {
            const int idx = tid + i * kAbsThreads, r = row_of(idx);
            if (idx < kTile * cpr) *(U4 *)(Cs + r * ldc + (idx - r * cpr) * 8) = pre[i];
        }
        __syncthreads();
        if (t + 1 < ntiles) {
            load_tile(t + 1, page_next);
            page_next = page_of(t + 2);
        }
        // ---- scores: this wave's 16 keys x 16 rows
        {
            const int kt = wave & 3, other = wave >> 2;
            const int qt = MT == 1 ? 0 : other;
            lf4_t s4 = {0.f, 0.f, 0.f, 0.f}, s5 = {0.f, 0.f, 0.f, 0.f};
            const T *ca = Cs + (kt * 16 + col) * ldc + quad * 8, *qb = Qs + (qt * 16 + col) * ldc + quad * 8;
            // (four steps at a time: their reads are in flight together; steps past the row multiply zeros)
            for (int k4 = MT == 1 ? other : 0; k4 < nks; k4 += 4 * KS) {
                U4 fa[4], fb[4];
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    const int ks = k4 + j * KS, kc = min(ks, nks - 1);
                    fa[j] = *(const U4 *)(ca + kc * 32);
                    fb[j] = *(const U4 *)(qb + kc * 32);
                    if (ks >= nks) fb[j] = U4{0u, 0u, 0u, 0u};
                }
                s4 = MfmaL16<T>::run(fa[0], fb[0], s4);
                s5 = MfmaL16<T>::run(fa[1], fb[1], s5);
                s4 = MfmaL16<T>::run(fa[2], fb[2], s4);
                s5 = MfmaL16<T>::run(fa[3], fb[3], s5);
            }
            s4 += s5;
            float *dst = Ss + ((MT == 1 ? other : 0) * 16 * MT + qt * 16 + col) * SST + kt * 16 + quad * 4;
            *(float4 *)dst = float4{s4[0], s4[1], s4[2], s4[3]};
        }
        __syncthreads();
        // ---- softmax of row `col` of every query tile, keys 32 * half + 8 * quad .. + 7 of the tile
        const int key0 = k0 + t * kTile + quad * 8;
        U4 ph[MT][2], pl[MT][2];
#pragma unroll
        for (int m = 0; m < MT; m++) {
            float sv[16];
            float tmax = -INFINITY;
#pragma unroll
            for (int hf = 0; hf < 2; hf++) {
                const float *src = Ss + (m * 16 + col) * SST + hf * 32 + quad * 8;
                float *v = sv + 8 * hf;
                *(float4 *)v = *(const float4 *)src;
                *(float4 *)(v + 4) = *(const float4 *)(src + 4);
                if constexpr (KS == 2) {
                    const float4 a = *(const float4 *)(src + 16 * MT * SST), c = *(const float4 *)(src + 16 * MT * SST + 4);
                    v[0] += a.x; v[1] += a.y; v[2] += a.z; v[3] += a.w;
                    v[4] += c.x; v[5] += c.y; v[6] += c.z; v[7] += c.w;
                }
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    v[e] = key0 + 32 * hf + e < bound[m] ? v[e] * p.scale : -INFINITY;
                    tmax = fmaxf(tmax, v[e]);
                }
            }
            tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
            tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
            const float m_new = fmaxf(m_run[m], tmax);
            float alpha = 1.f, psum = 0.f;
            if (m_new > -INFINITY) {
                alpha = fast_exp(m_run[m] - m_new);
#pragma unroll
                for (int e = 0; e < 16; e++) {
                    sv[e] = fast_exp(sv[e] - m_new);
                    psum += sv[e];
                }
            } else {
#pragma unroll
                for (int e = 0; e < 16; e++) sv[e] = 0.f;
            }
            m_run[m] = m_new;
            l_run[m] = l_run[m] * alpha + psum;
            if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
                for (int c = 0; c < CB; c++) {
                    acc[m][c][0] *= alpha;
                    acc[m][c][1] *= alpha;
                }
            }
            // the weights enter the product as a sum of two storage-type values
#pragma unroll
            for (int hf = 0; hf < 2; hf++) {
                float *v = sv + 8 * hf;
                ph[m][hf] = U4{pack2<T>(v[0], v[1]), pack2<T>(v[2], v[3]), pack2<T>(v[4], v[5]), pack2<T>(v[6], v[7])};
                float hi[8];
                widen8<T>(ph[m][hf], hi);
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] -= hi[e];
                pl[m][hf] = U4{pack2<T>(v[0], v[1]), pack2<T>(v[2], v[3]), pack2<T>(v[4], v[5]), pack2<T>(v[6], v[7])};
            }
        }
        // ---- O^T += C^T . P: a pair of neighbouring latents per dword, split into two operands by v_perm
#pragma unroll
        for (int c = 0; c < CB; c++) {
            const int blk = wave + kAbsWaves * c;
            if (blk < nblk) {
#pragma unroll
                for (int hf = 0; hf < 2; hf++) {
                    uint32_t w[8];
#pragma unroll
                    for (int i = 0; i < 8; i++) w[i] = *(const uint32_t *)(Cs + (hf * 32 + quad * 8 + i) * ldc + blk * 32 + col * 2);
                    const U4 ev = U4{__builtin_amdgcn_perm(w[1], w[0], 0x05040100u), __builtin_amdgcn_perm(w[3], w[2], 0x05040100u),
                                     __builtin_amdgcn_perm(w[5], w[4], 0x05040100u), __builtin_amdgcn_perm(w[7], w[6], 0x05040100u)};
                    const U4 od = U4{__builtin_amdgcn_perm(w[1], w[0], 0x07060302u), __builtin_amdgcn_perm(w[3], w[2], 0x07060302u),
                                     __builtin_amdgcn_perm(w[5], w[4], 0x07060302u), __builtin_amdgcn_perm(w[7], w[6], 0x07060302u)};
#pragma unroll
                    for (int m = 0; m < MT; m++) {
                        acc[m][c][0] = MfmaL16<T>::run(ev, ph[m][hf], acc[m][c][0]);
                        acc[m][c][1] = MfmaL16<T>::run(od, ph[m][hf], acc[m][c][1]);
                        acc[m][c][0] = MfmaL16<T>::run(ev, pl[m][hf], acc[m][c][0]);
                        acc[m][c][1] = MfmaL16<T>::run(od, pl[m][hf], acc[m][c][1]);
                    }
                }
            }
        }
    }
    // ---- partial results: lane (col, quad) holds latents 32 blk + 2 (4 quad + e) + par of row col
#pragma unroll
    for (int m = 0; m < MT; m++) {
        l_run[m] += __shfl_xor(l_run[m], 16, 64);
        l_run[m] += __shfl_xor(l_run[m], 32, 64);
        const int r = r0 + 16 * m + col;
        if (r >= nrows) continue;
        const size_t at = ((size_t)b * nrows + r) * p.nsplit + split;
#pragma unroll
        for (int c = 0; c < CB; c++) {
            const int blk = wave + kAbsWaves * c;
            if (blk < nblk) {
                float *dst = p.part_o + at * d.rp + blk * 32 + 8 * quad;
                *(float4 *)dst = float4{acc[m][c][0][0], acc[m][c][1][0], acc[m][c][0][1], acc[m][c][1][1]};
                *(float4 *)(dst + 4) = float4{acc[m][c][0][2], acc[m][c][1][2], acc[m][c][0][3], acc[m][c][1][3]};
            }
        }
        if (wave == 0 && quad == 0) {
            p.part_ml[at * 2] = m_run[m];
            p.part_ml[at * 2 + 1] = l_run[m];
        }
    }
}

// One workgroup per (query, head), f32 arithmetic throughout: scores of 256 keys at a time, one per thread, then the
// latents one per thread.
template <typename T>
__global__ __launch_bounds__(256) void latent_absorbed_plain_kernel(LatentParams p) {
    extern __shared__ __align__(16) char smem[];
    const LatentDims &d = p.d;
    const int lw = d.lw(), h = blockIdx.x, row = blockIdx.y, b = row / p.S, tid = threadIdx.x;
    float *q = (float *)smem, *o = q + lw, *pk = o + d.rp;  // [lw], [rp], [256]
    __shared__ float red[8];
    const int bound = *p.d_past + row % p.S + 1;
    const T *qa = (const T *)p.q_abs + ((size_t)row * d.H + h) * lw;
    for (int k = tid; k < lw; k += 256) q[k] = Elem<T>::ld(qa, k);
    for (int k = tid; k < d.rp; k += 256) o[k] = 0.f;
    float m_run = -INFINITY, l_run = 0.f;
    __syncthreads();
    for (int t0 = 0; t0 < bound; t0 += 256) {
        float s = -INFINITY;
        if (t0 + tid < bound) {
            const T *c = (const T *)p.cache + latent_row(p, b, t0 + tid) * lw;
            float a = 0.f;
            for (int k = 0; k < lw; k += 8) {
                float f[8];
                load8<T>(c + k, f);
#pragma unroll
                for (int e = 0; e < 8; e++) a = fmaf(q[k + e], f[e], a);
            }
            s = a * p.scale;
        }
        const float wm = wave_max(s);
        if ((tid & 63) == 0) red[tid >> 6] = wm;
        __syncthreads();
        const float m_new = fmaxf(m_run, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float alpha = expf(m_run - m_new), pe = expf(s - m_new);
        m_run = m_new;
        pk[tid] = pe;
        const float ws = wave_sum(pe);
        if ((tid & 63) == 0) red[4 + (tid >> 6)] = ws;
        __syncthreads();
        l_run = l_run * alpha + (red[4] + red[5] + red[6] + red[7]);
        const int n = min(256, bound - t0);
        for (int k = tid; k < d.rp; k += 256) {
            float a = 0.f;
            for (int j = 0; j < n; j++) a = fmaf(pk[j], Elem<T>::ld((const T *)p.cache, latent_row(p, b, t0 + j) * lw + k), a);
            o[k] = o[k] * alpha + a;
        }
        __syncthreads();
    }
    const size_t at = (size_t)row * d.H + h;
    for (int k = tid; k < d.rp; k += 256) p.part_o[at * d.rp + k] = o[k];
    if (tid == 0) {
        p.part_ml[at * 2] = m_run;
        p.part_ml[at * 2 + 1] = l_run;
    }
}

static bool absorbed_mfma_supported(const LatentDims &d, int dtype) { return dtype == MYNN_BF16 && d.rp <= 512 && d.rotp <= 128; }

// 16-row tiles per workgroup: one while there are few rows (more workgroups, each with less to do), else two per key read
static int absorbed_row_tiles(int B, int S, const LatentDims &d) { return S * d.H <= 16 || (long)B * S * d.H <= 64 ? 1 : 2; }

int latent_absorbed_splits(int B, int S, const LatentDims &d, int max_seq, int dtype) {
    if (!absorbed_mfma_supported(d, dtype)) return 1;
    const int mt = absorbed_row_tiles(B, S, d);
    const long tiles = (long)B * ((S * d.H + 16 * mt - 1) / (16 * mt));
    long n = 512 / tiles;
    const long most = (max_seq + kMinRange - 1) / kMinRange;
    n = n > 128 ? 128 : n;
    n = n > most ? most : n;
    return n < 1 ? 1 : (int)n;
}

int latent_attention_absorbed(const LatentParams &p, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.q_abs && p.cache && p.part_o && p.part_ml && p.nsplit >= 1, MYNN_ERR_INVALID, "latent attention: null operand");
    const LatentDims &d = p.d;
    MYNN_REQUIRE(!p.paging.table || (1 << p.paging.shift) >= kTile, MYNN_ERR_UNSUPPORTED, "latent attention: pages of %d rows", 1 << p.paging.shift);
    if (!absorbed_mfma_supported(d, dtype)) {
        MYNN_REQUIRE(p.nsplit == 1 && p.B * p.S <= 65535, MYNN_ERR_UNSUPPORTED, "latent attention: %d rows, %d ranges", p.B * p.S, p.nsplit);
        const size_t lds = (size_t)(d.lw() + d.rp + 256) * 4;
        MYNN_REQUIRE(lds <= 60 * 1024, MYNN_ERR_UNSUPPORTED, "latent attention: latent of %d values", d.rank);
        return dispatch_dense(dtype, [&](auto *t) {
            using T = std::remove_pointer_t<decltype(t)>;
            MYNN_LAUNCH(latent_absorbed_plain_kernel<T>, dim3(d.H, p.B * p.S), dim3(256), lds, s, p);
            return launch_status("latent_absorbed_plain_kernel");
        });
    }
    const int mt = absorbed_row_tiles(p.B, p.S, d);
    const unsigned cpr = d.lw() >> 3;
    const dim3 grid(p.nsplit, (p.S * d.H + 16 * mt - 1) / (16 * mt), p.B);
    MYNN_REQUIRE(grid.y <= 65535 && grid.z <= 65535, MYNN_ERR_UNSUPPORTED, "latent attention: %d rows of %d heads", p.S, d.H);
    const size_t lds = (size_t)(kTile + 16 * mt) * (d.lw() + 8) * 2 + (size_t)(mt == 1 ? 2 : 1) * 16 * mt * (kTile + 4) * 4;
    auto go = [&](auto kernel) {
        if (lds > 60 * 1024) MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        MYNN_LAUNCH(kernel, grid, dim3(kAbsThreads), lds, s, p, ((1u << 20) + cpr - 1) / cpr);
        return launch_status("latent_absorbed_kernel");
    };
    const bool wide = (d.rp >> 5) > kAbsWaves;
    if (mt == 1) return wide ? go(latent_absorbed_kernel<bf16_t, 1, 2>) : go(latent_absorbed_kernel<bf16_t, 1, 1>);
    return wide ? go(latent_absorbed_kernel<bf16_t, 2, 2>) : go(latent_absorbed_kernel<bf16_t, 2, 1>);
}

// ---- merge of the key ranges, W_uv, gate: NT / 8 value dimensions of one (query, head) per workgroup -----------------
constexpr int kMaxRanges = 128;
template <typename T, int NT>
__global__ __launch_bounds__(NT) void latent_out_kernel(LatentParams p) {
    extern __shared__ __align__(16) char smem[];
    float *o = (float *)smem;  // [rp], then the partial sums
    __shared__ float wgt[kMaxRanges];
    const LatentDims &d = p.d;
    const int h = blockIdx.y, row = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const size_t at = ((size_t)row * d.H + h) * p.nsplit;
    // Requested before the context length is known, so that the loads are one round trip: the ranges' maxima and sums, the
    // first kAhead ranges of the thread's four latents, and this wave's first eight rows of W_uv (a latent of up to 512
    // values: one piece per lane).  What lies past the last live range is not used.
    constexpr int kAhead = 8;
    const int n4 = d.rp >> 2, ng = NT / min(n4, NT), grp = tid / n4, c4_0 = tid - grp * n4;  // thread = (four latents, every ng-th range)
    const float *po = p.part_o + at * d.rp, *ml = p.part_ml + at * 2;
    float2 r_ml[kMaxRanges / 64];
    if (wave == 0) {
#pragma unroll
        for (int i = 0; i < kMaxRanges / 64; i++) r_ml[i] = *(const float2 *)(ml + 2 * min(lane + 64 * i, p.nsplit - 1));
    }
    float4 ahead[kAhead];
    if (grp < ng) {
#pragma unroll
        for (int j = 0; j < kAhead; j++) ahead[j] = *(const float4 *)(po + (size_t)min(grp + j * ng, p.nsplit - 1) * d.rp + c4_0 * 4);
    }
    const int v0 = blockIdx.x * (NT / 8) + wave * 8;
    const T *uv = (const T *)p.ukv + ((size_t)d.H * d.dimp + (size_t)h * d.vdimp + v0) * d.rp;
    const bool have = lane * 8 < d.rp;
    Row8<T> wr[8];
#pragma unroll
    for (int j = 0; j < 8; j++)
        if (have) wr[j].get(uv + (size_t)j * d.rp + lane * 8);
    // ranges that hold a key this row sees
    const int live = p.nsplit == 1 ? 1 : (*p.d_past + row % p.S) / latent_range(*p.d_past + p.S, p.nsplit) + 1;
    if (wave == 0) {
        float m = -INFINITY, l = 0.f, e[kMaxRanges / 64];
#pragma unroll
        for (int i = 0; i < kMaxRanges / 64; i++)
            if (lane + 64 * i < live) m = fmaxf(m, r_ml[i].x);
        m = wave_max(m);
#pragma unroll
        for (int i = 0; i < kMaxRanges / 64; i++) {
            e[i] = lane + 64 * i < live ? expf(r_ml[i].x - m) : 0.f;
            l += lane + 64 * i < live ? e[i] * r_ml[i].y : 0.f;
        }
        l = wave_sum(l);
#pragma unroll
        for (int i = 0; i < kMaxRanges / 64; i++) wgt[lane + 64 * i] = e[i] / l;
    }
    __syncthreads();
    float *acc_s = o + d.rp;  // [ng][rp]
    for (int c4 = c4_0; c4 < n4 && grp < ng; c4 += NT) {
        float4 a = float4{0.f, 0.f, 0.f, 0.f};
        for (int i0 = grp; i0 < live; i0 += kAhead * ng) {
            if (i0 != grp || c4 != c4_0) {
#pragma unroll
                for (int j = 0; j < kAhead; j++) ahead[j] = *(const float4 *)(po + (size_t)min(i0 + j * ng, live - 1) * d.rp + c4 * 4);
            }
#pragma unroll
            for (int j = 0; j < kAhead; j++)
                if (i0 + j * ng < live) {
                    const float w = wgt[i0 + j * ng];
                    a.x = fmaf(w, ahead[j].x, a.x); a.y = fmaf(w, ahead[j].y, a.y);
                    a.z = fmaf(w, ahead[j].z, a.z); a.w = fmaf(w, ahead[j].w, a.w);
                }
        }
        *(float4 *)(acc_s + grp * d.rp + c4 * 4) = a;
    }
    __syncthreads();
    for (int k = tid; k < d.rp; k += NT) {
        float a = 0.f;
        for (int i = 0; i < ng; i++) a += acc_s[i * d.rp + k];
        o[k] = a;
    }
    __syncthreads();
    const float g = sigmoidf(Elem<T>::ld((const T *)p.proj, (size_t)row * d.n_in() + d.qcols() + d.lw() + h));
    float acc[8];
#pragma unroll
    for (int j = 0; j < 8; j++) {
        acc[j] = 0.f;
        for (int c = lane * 8; c < d.rp; c += 512) {
            float f[8];
            if (c < 512) wr[j].widen(f);
            else load8<T>(uv + (size_t)j * d.rp + c, f);
#pragma unroll
            for (int e = 0; e < 8; e++) acc[j] = fmaf(f[e], o[c + e], acc[j]);
        }
    }
#pragma unroll
    for (int j = 0; j < 8; j++) {
        acc[j] = wave_sum(acc[j]);
        if (lane == j) Elem<T>::st((T *)p.out, (size_t)row * d.acols() + h * d.vdimp + v0 + j, acc[j] * g);
    }
}

int latent_merge_out(const LatentParams &p, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.out && p.part_o && p.part_ml && p.ukv && p.proj && p.nsplit >= 1 && p.nsplit <= kMaxRanges, MYNN_ERR_INVALID, "latent merge: bad operand");
    MYNN_REQUIRE(p.B * p.S <= 65535, MYNN_ERR_UNSUPPORTED, "latent merge: %d rows", p.B * p.S);
    const int nt = p.d.vdimp % 64 ? 256 : 512;
    const size_t lds = (size_t)(1 + nt / std::min(p.d.rp >> 2, nt)) * p.d.rp * 4;
    MYNN_REQUIRE(lds <= 60 * 1024, MYNN_ERR_UNSUPPORTED, "latent merge: latent of %d values", p.d.rank);
    return dispatch_dense(dtype, [&](auto *t) {
        using T = std::remove_pointer_t<decltype(t)>;
        const dim3 grid(p.d.vdimp / (nt / 8), p.d.H, p.B * p.S);
        if (nt == 512) MYNN_LAUNCH((latent_out_kernel<T, 512>), grid, dim3(512), lds, s, p);
        else MYNN_LAUNCH((latent_out_kernel<T, 256>), grid, dim3(256), lds, s, p);
        return launch_status("latent_out_kernel");
    });
}

// ---- expanded form ------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentParams p, int b, size_t total) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= total) return;
    const int cpr = p.d.lw() >> 3, r = (int)(i / cpr), c = (int)(i % cpr) * 8;
    const U4 v = *(const U4 *)((const T *)p.cache + latent_row(p, b, r) * p.d.lw() + c);
    if (c < p.d.rp) *(U4 *)((T *)p.c_rows + (size_t)r * p.d.rp + c) = v;
    else *(U4 *)((T *)p.rot_rows + (size_t)r * p.d.rotp + c - p.d.rp) = v;
}
int latent_gather(const LatentParams &p, int b, int L, int dtype, hipStream_t s) {
    MYNN_REQUIRE(dtype == MYNN_BF16 && p.c_rows && p.rot_rows && L > 0 && L <= p.max_seq, MYNN_ERR_INVALID, "latent gather: bad operand");
    const size_t total = (size_t)L * (p.d.lw() >> 3);
    MYNN_LAUNCH(latent_gather_kernel<bf16_t>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, s, p, b, total);
    return launch_status("latent_gather_kernel");
}

// Flash attention with query / key width up to DK and value width up to DV (rows beyond the real widths: zeros), WAVES
// waves of 32 query rows, 64-key tiles.  Per tile: S^T = K . Q^T (K from LDS, Q in registers), softmax with one query per
// lane, O^T += V^T . P^T with P in the registers the first product left it in (v_mfma_f32_32x32x16's result layout is the
// operand layout of the next product, keys in a permuted order that V^T follows).
template <typename T, int DK, int DV, int WAVES>
__global__ __launch_bounds__(64 * WAVES, WAVES == 4 ? 2 : 1) void latent_prefill_kernel(LatentParams p, int b, int past) {
    constexpr int NT = 64 * WAVES, KEYS = 64, LDK = DK + 8, LDV = KEYS + 4, KSTEPS = DK / 16, DT = DV / 32;
    constexpr int CHK = KEYS * DK / 8 / NT, CHV = KEYS * DV / 8 / NT;
    static_assert(KEYS * DK / 8 % NT == 0 && (CHV == 1 || CHV == 2 || CHV == 4), "whole pieces per thread");
    extern __shared__ __align__(16) uint16_t pl_smem[];
    uint16_t *Ks = pl_smem, *Vt = pl_smem + 2 * KEYS * LDK;
    const LatentDims &d = p.d;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, g = lane >> 5;
    const int h = blockIdx.x, S = p.S, dk = d.dk(), kvc = d.kvcols();
    const int q_blk = ((int)gridDim.y - 1 - (int)blockIdx.y) * 32 * WAVES;  // the blocks with the most keys first
    const int qrow = q_blk + wave * 32 + col, qrow_c = min(qrow, S - 1);
    const int my_bound = past + qrow_c + 1;
    const int wave_bound = past + min(q_blk + wave * 32 + 31, S - 1) + 1, wave_all = past + min(q_blk + wave * 32, S - 1) + 1;
    const int blk_bound = past + min(q_blk + 32 * WAVES - 1, S - 1) + 1;
    const int ntiles = (blk_bound + KEYS - 1) / KEYS;
    const T *kv = (const T *)p.kv, *rot = (const T *)p.rot_rows;

    // thread -> CHK pieces of 8 values of the K tile; CHV neighbouring keys of the same 8 value dimensions
    const int key0 = (tid / (DV / 8)) * CHV, dd = (tid % (DV / 8)) * 8;
    U4 rk[CHK], rv[CHV];
    auto load_tile = [&](int t) {
#pragma unroll
        for (int i = 0; i < CHK; i++) {
            const int idx = tid + i * NT, c = (idx % (DK / 8)) * 8;
            const int key = min(t * KEYS + idx / (DK / 8), blk_bound - 1);
            rk[i] = U4{0u, 0u, 0u, 0u};
            if (c < d.dimp) rk[i] = *(const U4 *)(kv + (size_t)key * kvc + h * d.dimp + c);
            else if (c < dk) rk[i] = *(const U4 *)(rot + (size_t)key * d.rotp + c - d.dimp);
        }
#pragma unroll
        for (int i = 0; i < CHV; i++) {
            const int key = min(t * KEYS + key0 + i, blk_bound - 1);
            rv[i] = U4{0u, 0u, 0u, 0u};
            if (dd < d.vdimp) rv[i] = *(const U4 *)(kv + (size_t)key * kvc + d.H * d.dimp + h * d.vdimp + dd);
        }
    };
    auto store_tile = [&](int buf) {
#pragma unroll
        for (int i = 0; i < CHK; i++) {
            const int idx = tid + i * NT;
            *(U4 *)&Ks[buf * KEYS * LDK + (idx / (DK / 8)) * LDK + (idx % (DK / 8)) * 8] = rk[i];
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            uint32_t w[CHV];
#pragma unroll
            for (int c = 0; c < CHV; c++) w[c] = i == 0 ? rv[c].x : i == 1 ? rv[c].y : i == 2 ? rv[c].z : rv[c].w;
            uint16_t *lo = &Vt[buf * DV * LDV + (dd + 2 * i) * LDV + key0], *hi = lo + LDV;
            if constexpr (CHV == 1) {
                *lo = (uint16_t)w[0];
                *hi = (uint16_t)(w[0] >> 16);
            } else if constexpr (CHV == 2) {
                *(uint32_t *)lo = __builtin_amdgcn_perm(w[1], w[0], 0x05040100u);
                *(uint32_t *)hi = __builtin_amdgcn_perm(w[1], w[0], 0x07060302u);
            } else {
                *(uint2 *)lo = uint2{__builtin_amdgcn_perm(w[1], w[0], 0x05040100u), __builtin_amdgcn_perm(w[3], w[2], 0x05040100u)};
                *(uint2 *)hi = uint2{__builtin_amdgcn_perm(w[1], w[0], 0x07060302u), __builtin_amdgcn_perm(w[3], w[2], 0x07060302u)};
            }
        }
    };

    load_tile(0);
    const size_t prow = (size_t)b * S + qrow_c;
    const T *Q = (const T *)p.proj + prow * d.n_in() + h * dk;
    U4 qf[KSTEPS];
#pragma unroll
    for (int ks = 0; ks < KSTEPS; ks++) {
        qf[ks] = U4{0u, 0u, 0u, 0u};
        if (16 * ks < dk) qf[ks] = *(const U4 *)(Q + 16 * ks + 8 * g);
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
        const uint16_t *Kb = Ks + buf * KEYS * LDK, *Vb = Vt + buf * DV * LDV;
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
                if (MASKED && k0 + 32 * hf + 8 * (e >> 2) + 4 * g + (e & 3) >= my_bound) s[hf][e] = -INFINITY;
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
    load_tile(min(1, ntiles - 1));
    __syncthreads();
    for (int t = 0; t < ntiles; t++) {
        // tile t is in LDS, tile t + 1 in registers; its buffer was released by the last barrier
        if (t + 1 < ntiles) store_tile((t + 1) & 1);
        load_tile(min(t + 2, ntiles - 1));
        const int k0 = t * KEYS;
        if (k0 + KEYS <= wave_all) tile(t & 1, k0, std::false_type{});
        else if (k0 < wave_bound) tile(t & 1, k0, std::true_type{});
        __syncthreads();
    }

    l += __shfl_xor(l, 32, 64);
    if (qrow < S) {
        const float gate = sigmoidf(Elem<T>::ld((const T *)p.proj, prow * d.n_in() + d.qcols() + d.lw() + h));
        T *out = (T *)p.out + prow * d.acols() + h * d.vdimp;
        const float f = gate / l;
#pragma unroll
        for (int t2 = 0; t2 < DT; t2++)
#pragma unroll
            for (int e4 = 0; e4 < 4; e4++) {
                const int c = 32 * t2 + 8 * e4 + 4 * g;
                if (c < d.vdimp) *(uint2 *)(out + c) = uint2{pack2<T>(o[t2][4 * e4 + 0] * f, o[t2][4 * e4 + 1] * f), pack2<T>(o[t2][4 * e4 + 2] * f, o[t2][4 * e4 + 3] * f)};
            }
    }
}

bool latent_expanded_supported(const LatentDims &d, int dtype) { return dtype == MYNN_BF16 && d.dk() <= 256 && d.vdimp <= 128; }

int latent_attention_expanded(const LatentParams &p, int b, int past, int dtype, hipStream_t s) {
    MYNN_REQUIRE(p.kv && p.rot_rows && p.proj && p.out && latent_expanded_supported(p.d, dtype), MYNN_ERR_INVALID, "latent prefill attention: bad operand");
    MYNN_REQUIRE(past >= 0 && past + p.S <= p.max_seq && b < p.B, MYNN_ERR_INVALID, "latent prefill attention: rows %d + %d of %d", past, p.S, p.max_seq);
    auto go = [&](auto kernel, int DK, int DV, int waves) {
        const size_t lds = ((size_t)2 * 64 * (DK + 8) + (size_t)2 * DV * 68) * 2;
        if (lds > 60 * 1024) MYNN_HIP(hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        MYNN_LAUNCH(kernel, dim3(p.d.H, (p.S + 32 * waves - 1) / (32 * waves)), dim3(64 * waves), lds, s, p, b, past);
        return launch_status("latent_prefill_kernel");
    };
    const int dk = p.d.dk();
    if (p.d.vdimp <= 64) {
        if (dk <= 96) return go(latent_prefill_kernel<bf16_t, 96, 64, 4>, 96, 64, 4);
        if (dk <= 192) return go(latent_prefill_kernel<bf16_t, 192, 64, 8>, 192, 64, 8);
        return go(latent_prefill_kernel<bf16_t, 256, 64, 8>, 256, 64, 8);
    }
    if (dk <= 96) return go(latent_prefill_kernel<bf16_t, 96, 128, 4>, 96, 128, 4);
    if (dk <= 192) return go(latent_prefill_kernel<bf16_t, 192, 128, 8>, 192, 128, 8);
    return go(latent_prefill_kernel<bf16_t, 256, 128, 8>, 256, 128, 8);
}

}  // namespace mynn
