// Token mixers with a state per sequence (recurrent.hip): a gated delta rule with a decay per head and key channel, and a
// matrix memory with exponential gates.  All of it f32 except the rows handed to the output projection.
#pragma once
#include "window_attention.h"

namespace mynn {

// state rows [dp] of key channels, one per value column: a column is its own recurrence given the keys, queries and gates
bool recurrent_dim_supported(int dp);
// several tokens: blocks of kRecurrentBlock tokens, key channels padded to whole operand tiles; floats of a portion's operands
constexpr int kRecurrentBlock = 16;
__host__ __device__ inline int recurrent_keys(int dp) { return dp <= 64 ? 64 : dp <= 128 ? 128 : dp <= 256 ? 256 : 512; }
size_t recurrent_block_floats(int B, int S, int H, int dp, bool delta);

struct DeltaParams {
    DeltaDims d;
    float eps;
    const float *proj;        // [B * S, n_in]: q | k | v | beta | low-rank parts
    const float *conv_w;      // [taps, conv()]
    const void *low_w;        // T [n_low(), low()]: rows of the decays over the decay part, rows of the gates over the gate part
    const void *a_log, *dt_bias, *norm;  // T [H], [H * dp], [vp]
    float *state;             // sequence b at state + b * state_stride: [H][v][dp], conv ring
    long state_stride;
    const int32_t *d_past;
    int B, S;
    void *out;                // T [B * S, acols()]
    // several tokens at a time: prepared operands of the recurrence
    float *qk;                // [B * S, 2 * G * dp] unit queries | keys
    float *v;                 // [B * S, H * vp]
    float *beta;              // [B * S, H]
    void *low;                // T [B * S, low()]
    float *dec;               // [B * S, n_low()]: decays | gates, as the second map leaves them
    float *blocks;            // recurrent_block_floats
    float *o;                 // [B * S, H * vp]
};
int delta_step(const DeltaParams &p, int dtype, hipStream_t s);      // one new token per sequence: all of the mixer between its projections
int delta_prepare(const DeltaParams &p, int dtype, hipStream_t s);   // convolutions, unit norms, beta; low
int delta_blocks(const DeltaParams &p, int dtype, hipStream_t s);    // decays; the operands of every block
int delta_recurrence(const DeltaParams &p, hipStream_t s);
int delta_out(const DeltaParams &p, int dtype, hipStream_t s);       // head norm and gate; the conv ring

struct MemoryParams {
    ParallelDims d;
    float cap, out_scale, eps, q_scale;
    const float *proj;        // [B * S, n_in]
    const void *i_bias, *f_bias, *norm;  // T [R], [R], [R * rvp]
    float *state;             // sequence b at state + b * state_stride
    long state_stride;
    const int32_t *d_past;
    int B, S;
    void *out;                // T [B * S, acols()], heads behind the attention's
    float *blocks;            // recurrent_block_floats
    float *gates;             // [B * S, R, 4]: what is kept, what is put in, exp(-maximum)
    float *o;                 // [B * S, R, pad4(rv + 1)]: unnormed read-out, then the normaliser's
};
// both mixers of a parallel layer: convolutions, norms, rotation and cache append of the attention; for one new token per
// sequence the whole memory step, else the memory's gates
int parallel_prepare(const WindowAttnParams &a, const MemoryParams &m, int dtype, hipStream_t s);
int memory_blocks(const MemoryParams &p, hipStream_t s);
int memory_recurrence(const MemoryParams &p, hipStream_t s);
int memory_out(const WindowAttnParams &a, const MemoryParams &p, int dtype, hipStream_t s);  // head norm and gate; the attention's conv ring

}  // namespace mynn
