// Attention over the last `window` tokens and a sequence's first keep_first (window_attention.hip): grouped queries, values
// that are the keys before norm and rotation, a short convolution over time in front of both.
#pragma once
#include "dense_load.h"
#include "dense.h"
#include "model_spec.h"

namespace mynn {

struct WindowAttnParams {
    ParallelDims d;
    int window, keep_first;   // window 0: every earlier token is visible
    float scale, out_scale, eps;
    int rot_dims;
    const float2 *rot;        // (cos, sin) [max_seq, rot_dims / 2]
    const float *proj;        // [B * S, n_in]
    const float *conv_w;      // [taps, conv()]
    const void *q_norm, *k_norm;  // T [H * dimp], [G * dimp]
    float *ring;              // [taps][conv()] of sequence b at ring + b * state_stride: column ch of position p in slot p % taps
    long state_stride;
    void *q;                  // T [B * S, H * dimp]
    void *cache;              // T [B, max_seq, row()] or pages: keys, then values, of every kv head
    KvPaging paging;
    const int32_t *d_past;
    int B, S, max_seq;
    void *out;                // T [B * S, acols()], head h at h * dimp, times out_scale
    float *part_o, *part_ml;  // [B * S * H, nsplit, dimp], [.., 2]
    int nsplit;
};

#ifdef __HIPCC__
// Channels ch .. ch + 3 of the short convolution at token s of a portion that starts at position `past`: tokens before the
// portion are in the ring.  Zeros before the sequence.
__device__ inline float4 short_conv4(const float *w, const float *proj, long ld, const float *ring, int ch, int channels, int taps, int s, int past) {
    float4 y = float4{0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < taps; j++) {
        const int back = taps - 1 - j, at = past + s - back;
        float4 u = float4{0.f, 0.f, 0.f, 0.f};
        if (s >= back) u = *(const float4 *)(proj - (long)back * ld + ch);
        else if (at >= 0) u = *(const float4 *)(ring + (size_t)(at % taps) * channels + ch);
        const float4 c = *(const float4 *)(w + (size_t)j * channels + ch);
        y.x = fmaf(c.x, u.x, y.x); y.y = fmaf(c.y, u.y, y.y); y.z = fmaf(c.z, u.z, y.z); y.w = fmaf(c.w, u.w, y.w);
    }
    return y;
}

__device__ inline size_t window_cache_row(const WindowAttnParams &p, int b, int r) { return kv_cache_row(p.paging, b, 0, r, 1, p.max_seq); }

// q (which 0) or k and v (which 1) of one row: convolution, norm over all heads, rotation; NT threads, `buf` of a value per
// channel.  One new token per sequence: its projected values go into the ring too (their slot is not among those read).
template <typename T, int NT>
__device__ inline void window_prepare_row(const WindowAttnParams &p, int row, int which, float *buf, float *red) {
    const ParallelDims &d = p.d;
    const int b = row / p.S, s = row % p.S, past = *p.d_past, pos = past + s, tid = threadIdx.x;
    const int heads = which ? d.G : d.H, nch = heads * d.dimp, col0 = which ? d.H * d.dimp : 0, channels = d.conv();
    const float *proj = p.proj + (size_t)row * d.n_in();
    float *ring = p.ring + (size_t)b * p.state_stride;
    T *dst = which ? (T *)p.cache + window_cache_row(p, b, pos) * d.row() : (T *)p.q + (size_t)row * d.qcols();
    float ss = 0.f;
    for (int c = tid * 4; c < nch; c += NT * 4) {
        const float4 y = short_conv4(p.conv_w, proj, d.n_in(), ring, col0 + c, channels, d.taps, s, past);
        if (p.S == 1) *(float4 *)(ring + (size_t)(pos % d.taps) * channels + col0 + c) = *(const float4 *)(proj + col0 + c);
        if (which) store4<T>(dst + d.G * d.dimp + c, y);
        *(float4 *)(buf + c) = y;
        ss = fmaf(y.x, y.x, fmaf(y.y, y.y, fmaf(y.z, y.z, fmaf(y.w, y.w, ss))));
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; w++) t += red[w];
    const float inv = 1.0f / sqrtf(t / (float)(heads * d.dim) + p.eps);
    const T *nw = (const T *)(which ? p.k_norm : p.q_norm);
    const int half = p.rot_dims / 2;
    for (int c = tid * 4; c < nch; c += NT * 4) {
        const int i = c % d.dimp / 2;
        float4 x = *(const float4 *)(buf + c);
        Load4<T> wl;
        wl.get(nw + c);
        float f[4];
        wl.widen(f);
        x.x *= inv * f[0]; x.y *= inv * f[1]; x.z *= inv * f[2]; x.w *= inv * f[3];
        const float2 *cs = p.rot + (size_t)pos * half;
        if (i < half) {
            const float2 t2 = cs[i];
            x = float4{x.x * t2.x - x.y * t2.y, x.y * t2.x + x.x * t2.y, x.z, x.w};
        }
        if (i + 1 < half) {
            const float2 t2 = cs[i + 1];
            x = float4{x.x, x.y, x.z * t2.x - x.w * t2.y, x.w * t2.x + x.z * t2.y};
        }
        store4<T>(dst + c, x);
    }
}
#endif

// one query row at a time (decode; f32; shapes without a tile form): key ranges, then their merge when there are several
int window_attention_rows(const WindowAttnParams &p, int dtype, hipStream_t s);
int window_attention_merge(const WindowAttnParams &p, int dtype, hipStream_t s);
int window_attention_splits(int B, int S, const ParallelDims &d, int window, int keep_first, int max_seq);
bool window_attention_dim_supported(int dimp);
// prompts on the matrix cores; past: the portion's first position
bool window_prefill_supported(const ParallelDims &d, int dtype);
int window_attention_prefill(const WindowAttnParams &p, int past, int dtype, hipStream_t s);

}  // namespace mynn
