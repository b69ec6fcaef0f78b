// Linear algebra and row operators of executors that keep a 32-bit residual stream and weights in the storage type
// (dense.hip).  T is the storage type of weights and activations (bf16, or f32 throughout); every row extent is a
// multiple of 64 with zeros behind the last real value.
#pragma once
#include "kernels.h"

namespace mynn {

template <typename F> inline int dispatch_dense(int dt, F &&f) {
    switch (dt) {
    case MYNN_F32: return f((float *)nullptr);
    case MYNN_BF16: return f((bf16_t *)nullptr);
    default: return fail(MYNN_ERR_UNSUPPORTED, "dtype %d: this kernel is built for bf16 and f32", dt);
    }
}

// dst block copy: element (h, j, c) of H row blocks of `rows` rows and `cols` columns in CB column blocks; a row block
// starts every dst_rs / src_rs rows, a column block every dst_cs / src_cs columns.  group > 0: destination row r is
// written to (r / group) * 2 * group + which * group + r % group.
struct PackBlocks {
    void *dst;
    const void *src;
    long ldd, lds;
    int H, rows, dst_row0, dst_rs, src_row0, src_rs;
    int CB, cols, dst_col0, dst_cs, src_cs;
    int group, which;
};
int pack_blocks(const PackBlocks &p, int dtype, hipStream_t s);

// f32 weights of a short convolution, tap by tap: dst[j * channels + ch0 + h * dimp + i] = src[(h * dim + i) * taps + j]
struct PackTaps {
    float *dst;
    const void *src;
    int channels, ch0, heads, dim, dimp, taps;
};
int pack_taps(const PackTaps &p, int dtype, hipStream_t s);

// x[row] = table[id] (+ pair[hash of (previous id, id)]) as f32 [rows, ld]; row b * S + s is token past + s of sequence b.
// The ids are recorded in `history` (a cache row per token), where the previous id of a step's first token is found.
struct EmbedParams {
    float *x, *x0;           // x0: a second copy (may be null)
    const void *table, *pair;
    int64_t buckets, mul_prev, mul_cur;  // buckets == 0: no pair table
    const int64_t *ids;      // [B, S]
    const int32_t *d_past;
    int32_t *history;        // [B, max_seq] or pool pages
    KvPaging paging;
    int B, S, width, ld, vocab, max_seq;
};
int embed_tokens(const EmbedParams &p, int dtype, hipStream_t s);

// What precedes a linear: the sublayer output y still to be added to the residual stream, and the norm of the result.
//   x' = x + y_mul * rms_norm(y, wb)      (y null: x' = x)
//   RESIDUAL_NORM: act = rms_norm(x', wa);  RESIDUAL_CONCAT: act = [x', x0];  RESIDUAL: act = x';  ROWS: act is a row of T
//   already.  A norm's weight is w_add + the stored one.
enum { PRO_ROWS = 0, PRO_RESIDUAL_NORM = 1, PRO_RESIDUAL_CONCAT = 2, PRO_RESIDUAL = 3 };
struct ResidualNorm {
    const float *x;
    const void *y, *wb;
    float *x_out;            // receives x' (may be null; must differ from x in a GEMV, where every workgroup reads x)
    const void *wa;
    const float *x0;
    float eps;
    int width, ld;           // row extent and its padded form
    float w_add = 0.f, y_mul = 1.f;
};
// act[i] <- row first + i * stride of the stream, i < count; act has ld (CONCAT: 2 ld) columns
int residual_norm_rows(void *act, const ResidualNorm &r, int pro, int first, int stride, int count, int dtype, hipStream_t s);

// one row: out = store(w . act); w [N, K] T, K a multiple of 64.  store: DENSE_T (T), DENSE_F32 (f32, times *scale when
// given), DENSE_GEGLU (rows interleaved gate/up in groups of 32: out[N / 2] = T(gelu_tanh(gate) * up)).
// PRO_ROWS: act = T [K]; else r describes the row (K = ld or 2 ld).
enum { DENSE_T = 0, DENSE_F32 = 1, DENSE_GEGLU = 2 };
bool dense_gemv_supported(int K);
// cand (DENSE_F32): every workgroup leaves its largest output there, *n_cand of them (at most kGreedyCands); greedy_pick
// takes the best, the last maximum as argmax_rows does, and moves the loop state on.
struct GreedyCand {
    float value;
    int index;  // -1: none
};
constexpr int kGreedyCands = 1024;
int dense_gemv(void *out, const void *act, const ResidualNorm *r, int pro, const void *w, int N, int K, int store, const float *scale,
               int dtype, hipStream_t s, GreedyCand *cand = nullptr, int *n_cand = nullptr);
int greedy_pick(int32_t *out, const GreedyCand *cand, int n, AdvanceState adv, hipStream_t s);

// any number of rows: act [M, K]; 16-bit types on the matrix cores' 16-bit product, f32 on their f32 product
int dense_gemm(void *out, const void *act, const void *w, int M, int N, int K, int store, const float *scale, int dtype, hipStream_t s);

}  // namespace mynn
