// Loads and stores of a few storage-type values as f32, for 16-bit types and f32 alike.
#pragma once
#include "mfma.h"

namespace mynn {

// four values of T, kept as loaded until they are used
template <typename T> struct Load4 {
    uint2 v;
    __device__ void get(const T *p) { v = *(const uint2 *)p; }
    __device__ void widen(float *f) const {
        const T *h = (const T *)&v;
#pragma unroll
        for (int i = 0; i < 4; i++) f[i] = Elem<T>::ld(h, i);
    }
};
template <> struct Load4<float> {
    float4 v;
    __device__ void get(const float *p) { v = *(const float4 *)p; }
    __device__ void widen(float *f) const { f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w; }
};
template <typename T> __device__ inline void store4(T *p, const float4 &v) { *(uint2 *)p = uint2{pack2<T>(v.x, v.y), pack2<T>(v.z, v.w)}; }
template <> __device__ inline void store4<float>(float *p, const float4 &v) { *(float4 *)p = v; }

// the 16 / sizeof(T) values of one 16-byte load
template <typename T> __device__ inline void widen16b(const U4 &v, float *f) { widen8<T>(v, f); }
template <> __device__ inline void widen16b<float>(const U4 &v, float *f) { *(float4 *)f = __builtin_bit_cast(float4, v); }
// eight values at an address aligned to their size
template <typename T> __device__ inline void load8(const T *p, float *f) { widen8<T>(*(const U4 *)p, f); }
template <> __device__ inline void load8<float>(const float *p, float *f) {
    *(float4 *)f = *(const float4 *)p;
    *(float4 *)(f + 4) = *(const float4 *)(p + 4);
}

// eight values of T, kept as loaded until they are used
template <typename T> struct Row8 {
    U4 v;
    __device__ void get(const T *p) { v = *(const U4 *)p; }
    __device__ void widen(float *f) const { widen8<T>(v, f); }
};
template <> struct Row8<float> {
    float4 a, b;
    __device__ void get(const float *p) { a = *(const float4 *)p; b = *(const float4 *)(p + 4); }
    __device__ void widen(float *f) const { *(float4 *)f = a; *(float4 *)(f + 4) = b; }
};

__device__ inline float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh(u)) = z * sigmoid(2 u), u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ inline float gelu_tanh_arg(float z) { return 1.5957691216057308f * fmaf(0.044715f * z * z, z, z); }
__device__ inline float gelu_tanh(float z) { return z * sigmoidf(gelu_tanh_arg(z)); }

}  // namespace mynn
