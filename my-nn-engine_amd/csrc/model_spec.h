// What a config.json says about a model: the registry's description of a decoder (model_registry.hip).
#pragma once
#include <memory>
#include <string>
#include <unordered_map>
#include <vector>

#include "mynn_common.h"

namespace mynn {

// Rotary positions: pair i of `dims` dimensions turns by position * frequency(i), base^(-2i / dims) unless scaled.
// Scaled (the Llama 3.1 rule): wavelengths above original / low are stretched by `factor`, those below original / high are
// kept, and in between the two blend.
struct RotarySpec {
    double base = 10000.0;
    int dims = 0;
    bool scaled = false;
    double factor = 1.0, low = 1.0, high = 1.0, original = 0.0;
    double frequency(int i) const;
    bool operator==(const RotarySpec &o) const {
        return base == o.base && dims == o.dims && scaled == o.scaled && (!scaled || (factor == o.factor && low == o.low && high == o.high && original == o.original));
    }
};

// Grouped-query attention whose values are the keys before norm and rotation: q and k pass a causal convolution of `taps`
// tokens per channel, one norm over all heads, and a rotation; a query sees the last `window` tokens (0: all) and the
// sequence's first keep_first.
struct WindowAttentionSpec {
    int heads = 0, kv_heads = 0, dim = 0, taps = 1, window = 0, keep_first = 0;
    float scale = 1.f;
    RotarySpec rot;
};
// Matrix memory: per head a state [dim, vdim] and a normaliser [dim] with exponential input and forget gates, whose
// logarithms are soft-capped at gate_cap.
struct MatrixMemorySpec {
    int heads = 0, dim = 0, vdim = 0;
    float gate_cap = 1.f;
};
// Gated delta rule with one decay per head and key channel; decays and output gates come through low-rank maps.
struct ChannelDeltaSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1, decay_rank = 0, gate_rank = 0;
};

// A token mixer of a layer.  LATENT_ATTENTION: keys and values of every head are linear images of one normed latent per
// token (kv_rank values) plus one rotated key part shared by the heads, so a token's cache row is the latent and that part.
// PARALLEL: left_scale * window attention + right_scale * matrix memory, both of the same input.
struct MixerSpec {
    enum Kind { LATENT_ATTENTION, PARALLEL, CHANNEL_DELTA } kind = LATENT_ATTENTION;
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0;
    float scale = 1.f;
    RotarySpec rot;
    WindowAttentionSpec window;
    MatrixMemorySpec memory;
    float left_scale = 1.f, right_scale = 1.f;
    ChannelDeltaSpec delta;
};

// A feed-forward.  GATED_DENSE: down(act(gate h) * up h).  EXPERTS: `top` of `experts` such maps, the ones with the largest
// sigmoid scores, each over the input times its score.
struct MlpSpec {
    enum Kind { NONE, GATED_DENSE, EXPERTS } kind = NONE;
    int ff = 0, experts = 0, top = 0;
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

// One execution of a layer: a looped layer has several, each with a cache and a state of its own.
struct LayerRun {
    int layer;
    bool starts_pass;
    int cache = -1, memory = -1;  // its buffers among ModelSpec::states (-1: it has none)
};

// A buffer of a session's state: a row per token (row_elems values of the storage type, or row_bytes), or a block per
// sequence that stands for everything read so far (seq_floats f32 values).
struct StateSpec {
    size_t row_elems = 0, row_bytes = 0, seq_floats = 0;
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
    // norms of a layer: in front of its sublayers (norm1, norm2) and behind them (norm1b, norm2b), or behind them only
    // (norm1, norm2); a norm's weight is norm_offset + the stored one; a sublayer's output enters the sum times residual_mult
    bool pre_norm = true;
    float norm_offset = 0.f, residual_mult = 1.f;
    std::vector<LayerRun> runs;         // in execution order
    std::vector<StateSpec> states;      // in the order of `session_state`
    int history = -1;                   // the token history among them
    bool sequence_state() const {
        for (const StateSpec &s : states)
            if (s.seq_floats) return true;
        return false;
    }
    std::vector<TensorSpec> tensors;    // the checkpoint's tensors, in the order of `initializer`
    std::unordered_map<std::string, int> tensor_at;
    int tensor_index(const std::string &name) const {
        auto it = tensor_at.find(name);
        return it == tensor_at.end() ? -1 : it->second;
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


// Columns of the projections and state of a window attention beside a matrix memory: attention heads padded to 32 (the
// matrix cores' step), memory heads to 4 (one 16-byte load).
struct ParallelDims {
    int H, G, dim, dimp, taps;      // attention
    int R, rd, rdp, rv, rvp;        // memory
    __host__ __device__ int qcols() const { return H * dimp; }
    __host__ __device__ int conv() const { return (H + G) * dimp; }       // convolved channels: q | k, the first columns
    __host__ __device__ int mem_q() const { return conv(); }
    __host__ __device__ int mem_k() const { return mem_q() + R * rdp; }
    __host__ __device__ int mem_v() const { return mem_k() + R * rdp; }
    __host__ __device__ int mem_g() const { return mem_v() + R * rvp; }
    __host__ __device__ int mem_i() const { return mem_g() + R * rvp; }
    __host__ __device__ int mem_f() const { return mem_i() + pad_to(R, 4); }
    __host__ __device__ int n_in() const { return pad_to(mem_f() + R, 64); }
    __host__ __device__ int acols() const { return pad_to(H * dimp + R * rvp, 64); }  // attention heads | memory heads
    __host__ __device__ int row() const { return 2 * G * dimp; }          // cache row: keys, values
    // state of a sequence: memory columns [R][rv + 1][rdp] (the last one is the normaliser), running maxima, conv ring
    __host__ __device__ int st_max() const { return R * (rv + 1) * rdp; }
    __host__ __device__ int st_ring() const { return st_max() + pad_to(R, 4); }
    __host__ __device__ int state() const { return st_ring() + taps * conv(); }
};
inline ParallelDims parallel_dims(const MixerSpec &m) {
    const WindowAttentionSpec &a = m.window;
    const MatrixMemorySpec &r = m.memory;
    return ParallelDims{a.heads, a.kv_heads, a.dim, pad_to(a.dim, 32), a.taps, r.heads, r.dim, pad_to(r.dim, 4), r.vdim, pad_to(r.vdim, 4)};
}

struct DeltaDims {
    int H, G, d, dp, v, vp, taps, ra, rg, rap, rgp;
    __host__ __device__ int col_k() const { return G * dp; }
    __host__ __device__ int col_v() const { return 2 * G * dp; }
    __host__ __device__ int conv() const { return 2 * G * dp + H * vp; }  // convolved channels: q | k | v
    __host__ __device__ int col_b() const { return conv(); }
    __host__ __device__ int col_low() const { return pad_to(col_b() + H, 4); }        // low-rank parts of decay and gate
    __host__ __device__ int low() const { return rap + rgp; }
    __host__ __device__ int n_in() const { return pad_to(col_low() + low(), 64); }
    __host__ __device__ int n_low() const { return H * (dp + vp); }       // what the second map makes: decays | gates
    __host__ __device__ int acols() const { return pad_to(H * vp, 64); }
    // state of a sequence: [H][v][dp], conv ring
    __host__ __device__ int st_ring() const { return H * v * dp; }
    __host__ __device__ int state() const { return st_ring() + taps * conv(); }
};
inline DeltaDims delta_dims(const ChannelDeltaSpec &m) {
    return DeltaDims{m.heads, m.kv_heads, m.dim, pad_to(m.dim, 4), m.vdim, pad_to(m.vdim, 4), m.taps,
                     m.decay_rank, m.gate_rank, pad_to(m.decay_rank, 64), pad_to(m.gate_rank, 64)};
}

}  // namespace mynn
