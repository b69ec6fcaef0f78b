// What a config.json says about a model: the registry's description of a decoder (model_registry.hip).
#pragma once
#include <memory>
#include <string>
#include <vector>

#include "mynn_common.h"

namespace mynn {

// Rotary positions: pair i of `dims` dimensions turns by position * base^(-2i / dims).
struct RotarySpec {
    double base = 10000.0;
    int dims = 0;
};

// A token mixer of a layer.  LATENT_ATTENTION: keys and values of every head are linear images of one normed latent per
// token (kv_rank values) plus one rotated key part shared by the heads, so a token's cache row is the latent and that part.
struct MixerSpec {
    enum Kind { LATENT_ATTENTION } kind = LATENT_ATTENTION;
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0;
    float scale = 1.f;
    RotarySpec rot;
};

// A feed-forward: down(act(gate h) * up h)
struct MlpSpec {
    enum Kind { NONE, GATED_DENSE } kind = NONE;
    int ff = 0;
};

struct LayerSpec {
    MixerSpec mixer;
    MlpSpec mlp;
};

// Layers [start, stop) run `times` times in a row with the same weights; a pass starts with a linear map of [x; x0]
struct LoopSpec {
    int start = 0, stop = 0, times = 0;  // times == 0: no loop
};

// Row (previous * mul_prev + current * mul_cur) mod buckets of a second embedding table; the extra last row for a
// sequence's first token
struct BigramSpec {
    int64_t buckets = 0, mul_prev = 0, mul_cur = 0;  // buckets == 0: no such table
};

struct TensorSpec {
    std::string name;
    std::vector<int64_t> shape;
    size_t elements() const {
        size_t n = 1;
        for (int64_t d : shape) n *= (size_t)d;
        return n;
    }
};

// One execution of a layer: a looped layer has several, each with a cache of its own.
struct LayerRun {
    int layer;
    bool starts_pass;
};

struct ModelSpec {
    enum Family { LLAMA, LAYERED } family = LLAMA;
    std::string architecture;
    int vocab = 0, width = 0;
    float eps = 1e-6f;
    // LLAMA: the fixed graph's configuration (executor fields left 0)
    mynn_model_config llama{};
    // LAYERED
    float logit_scale = 1.f;
    BigramSpec bigram;
    std::vector<LayerSpec> layers;
    LoopSpec loop;
    std::vector<LayerRun> runs;         // in execution order
    std::vector<TensorSpec> tensors;    // the checkpoint's tensors, in the order of `initializer`
    int tensor_index(const std::string &name) const {
        for (size_t i = 0; i < tensors.size(); i++)
            if (tensors[i].name == name) return (int)i;
        return -1;
    }
};

// the description behind an arch id (mynn_arch_open); nullptr for an unknown id
std::shared_ptr<const ModelSpec> arch_spec(int arch);

// ---- padded extents of the layered executor: every dimension a kernel walks is a multiple of its tile, the rest zeros
__host__ __device__ inline int pad_to(int v, int a) { return (v + a - 1) / a * a; }
struct LatentDims {
    int H, dim, rot, vdim, rank;         // as configured
    int dimp, rotp, vdimp, rp;           // padded: head parts to 32, the latent to 64
    __host__ __device__ int dk() const { return dimp + rotp; }   // a query's / key's width
    __host__ __device__ int lw() const { return rp + rotp; }     // a cache row: latent, then the rotated part
    __host__ __device__ int qcols() const { return H * dk(); }
    __host__ __device__ int n_in() const { return qcols() + lw() + pad_to(H, 8); }  // q | latent | rotated part | gates
    __host__ __device__ int kvcols() const { return H * (dimp + vdimp); }           // expanded keys and values of a token
    __host__ __device__ int acols() const { return pad_to(H * vdimp, 64); }         // attention output row
};
inline LatentDims latent_dims(const MixerSpec &m) {
    return LatentDims{m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank,
                      pad_to(m.dim, 32), pad_to(m.rot_dim, 32), pad_to(m.vdim, 32), pad_to(m.kv_rank, 64)};
}

}  // namespace mynn
