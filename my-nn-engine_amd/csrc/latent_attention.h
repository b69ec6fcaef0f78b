// Latent attention (latent_attention.hip): a token's cache row is a normed latent c [rp] and one rotated key part [rotp]
// shared by all heads; key and value of head h are W_uk[h] c and W_uv[h] c.
#pragma once
#include "dense.h"
#include "model_spec.h"

namespace mynn {

struct LatentParams {
    LatentDims d;
    float scale, eps;
    int rot_dims;             // rotated dimensions of the rot part (pairs 2i, 2i + 1)
    const float2 *rot;        // (cos, sin) [max_seq, rot_dims / 2]
    void *proj;               // T [B * S, n_in]: q | latent | rotated part | gates, from the input projection
    const void *norm_w;       // T [rp]
    const void *ukv;          // T [kvcols, rp]: key rows of all heads, then value rows
    void *cache;              // T [B, max_seq, lw], or pages [n_pages, P, lw]
    KvPaging paging;
    const int32_t *d_past;
    int B, S, max_seq;
    void *out;                // T [B * S, acols]: the gated head outputs
    // absorbed form: queries taken into the latent space, partial results per key range
    void *q_abs;              // T [B * S, H, lw]
    float *part_o, *part_ml;  // [B * S * H, nsplit, rp], [.., 2]
    int nsplit;
    // expanded form: keys and values of every visible token, made per layer (one sequence at a time)
    void *c_rows, *rot_rows, *kv;  // T [max_seq, rp], [max_seq, rotp], [max_seq, kvcols]
};

// latent norm, rotation and cache append of the step's tokens; ABSORB: the queries go to q_abs, else they are rotated
// in place
int latent_prepare(const LatentParams &p, bool absorb, int dtype, hipStream_t s);
// absorbed form (any number of query rows): attention over the cached rows, then merge, W_uv and gate
int latent_attention_absorbed(const LatentParams &p, int dtype, hipStream_t s);
int latent_merge_out(const LatentParams &p, int dtype, hipStream_t s);
int latent_absorbed_splits(int B, int S, const LatentDims &d, int max_seq, int dtype);
// expanded form (bf16, prompts): gather the first L cache rows of sequence b; attention of its S queries over kv
bool latent_expanded_supported(const LatentDims &d, int dtype);
int latent_gather(const LatentParams &p, int b, int L, int dtype, hipStream_t s);
int latent_attention_expanded(const LatentParams &p, int b, int past, int dtype, hipStream_t s);

}  // namespace mynn
