// The layered executor's own state and the pieces its mixers and feed-forwards share (layered.hip: skeleton, latent attention;
// layered_mixers.hip: recurrent mixers, window attention, experts).
#pragma once
#include <string>

#include "executor.h"
#include "experts.h"
#include "latent_attention.h"
#include "recurrent.h"

namespace mynn {

// a linear's rows in the storage type, padded [N, K]
struct DenseW {
    void *w = nullptr;
    int N = 0, K = 0;
};
struct LayerWeights {
    void *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr;
    DenseW in, o;                         // a mixer's projections
    void *latent_norm = nullptr;          // latent attention
    DenseW ukv;
    float *taps = nullptr;                // short convolutions
    void *q_norm = nullptr, *k_norm = nullptr, *head_norm = nullptr, *i_bias = nullptr, *f_bias = nullptr;
    DenseW low;                           // delta rule: second maps of decays and gates
    void *a_log = nullptr, *dt_bias = nullptr;
    DenseW gu, down, router;              // feed-forward; experts: one after another
};
struct LayeredWeights {
    std::vector<LayerWeights> layers;
    DenseW loop_in, head;
    void *final_norm = nullptr;
    std::vector<void *> owned;
    bool ready = false;
};

struct LayeredNet {
    std::shared_ptr<const ModelSpec> spec;
    const LayeredWeights *w = nullptr;
    const void *embed = nullptr, *bigram = nullptr;  // the caller's tables
    std::vector<void *> caches;   // per run (null: none)
    std::vector<float *> memory;  // per run: the sequence state (null: none)
    int32_t *history = nullptr;
    char *saved = nullptr;        // a copy of the sequence states (executor_save_state)
    std::vector<float2 *> rot;    // per layer, into rot_tables
    std::vector<void *> rot_tables;
    int ld = 0;                   // padded width
    float *xa = nullptr, *xb = nullptr, *x0 = nullptr, *logit_scale = nullptr;
    void *act = nullptr, *proj = nullptr, *attn = nullptr, *y = nullptr, *hmid = nullptr, *q_abs = nullptr;
    void *c_rows = nullptr, *rot_rows = nullptr, *kv = nullptr;
    float *part_o = nullptr, *part_ml = nullptr;
    GreedyCand *cand = nullptr;
    bool gemv = false;            // every linear fits the one-row kernel
    // recurrent mixers and window attention
    void *q = nullptr, *low = nullptr;
    float *gates = nullptr, *o = nullptr, *qk = nullptr, *v = nullptr, *beta = nullptr, *dec = nullptr, *blocks = nullptr;
    // experts
    float *router = nullptr, *score = nullptr, *parts = nullptr;
    int32_t *chosen = nullptr, *choice = nullptr, *tile_group = nullptr, *slot = nullptr;
    void *hsort = nullptr;
};

// padded weight copies, made once per weight set
struct WeightPacker {
    Model &m;
    LayeredWeights &w;
    const ModelSpec &s;
    int dt, ld;
    int alloc(void **p, size_t rows, size_t cols, size_t elem = 0);
    const void *src(const std::string &name) const {
        const int i = s.tensor_index(name);
        return i < 0 ? nullptr : m.wset->initializer[i];
    }
    int linear(DenseW &l, int N, int K) {
        l.N = N;
        l.K = K;
        return alloc(&l.w, N, K);
    }
    // `heads` blocks of n values, each padded to np
    int vec(void **p, const std::string &name, int heads, int n, int np, int padded);
    int norm(void **p, const std::string &name, int n, int padded) { return vec(p, name, 1, n, n, padded); }
    // rows of `heads` blocks of n rows (a block every np rows of dst, from row0) over K columns of the width
    int rows(DenseW &l, const std::string &name, int heads, int n, int np, int row0);
    // an output projection: heads * n columns of `name`, a block every np columns from col0
    int cols(DenseW &l, const std::string &name, int heads, int n, int np, int col0);
};
int pack_parallel(WeightPacker &pk, LayerWeights &o, const MixerSpec &mix, const std::string &mx);
int pack_channel_delta(WeightPacker &pk, LayerWeights &o, const MixerSpec &mix, const std::string &mx);
int pack_experts(WeightPacker &pk, LayerWeights &o, const MlpSpec &mlp, const std::string &p);

// bytes of the buffers the mixers need, the most of any layer
struct MixerScratch {
    size_t proj = 0, attn = 0, part_o = 0, part_ml = 0;
    size_t q = 0, low = 0, gates = 0, o = 0, qk = 0, v = 0, beta = 0, dec = 0, blocks = 0;
    size_t hmid = 0, router = 0, score = 0, parts = 0, chosen = 0, choice = 0, tile_group = 0, slot = 0, hsort = 0;
};
void scratch_recurrent(MixerScratch &x, const MixerSpec &mix, const mynn_model_config &c);
void scratch_experts(MixerScratch &x, const MlpSpec &mlp, const mynn_model_config &c, int ld);
int check_mixer(const MixerSpec &mix);

// The residual stream of the step in flight: the current rows, and the sublayer output that the next linear's prologue
// still has to norm and add.
struct Stream {
    Model &m;
    LayeredNet &n;
    int rows;
    bool one;  // one row: the prologue rides on the linear (dense_gemv), which writes the sum to the other buffer
    float *x, *other;
    const void *y = nullptr, *wb = nullptr;

    ResidualNorm row(const void *wa) const {
        return ResidualNorm{x, y, wb, y ? (one ? other : x) : nullptr, wa, n.x0, n.spec->eps, n.spec->width, n.ld, n.spec->norm_offset, n.spec->residual_mult};
    }
    void added() {
        if (y && one) std::swap(x, other);
        y = wb = nullptr;
    }
    double row_bytes(double eb) const { return n.ld * (4 + (y ? 4 + 2 * eb : 0)); }
};
int linear(Stream &s, void *out, const DenseW &w, int store, const char *name, const char *gemv_name, const void *act, const void *wa, int pro);
// leave the sublayer output in n.y
int run_parallel(Stream &st, int run, const LayerWeights &w, const MixerSpec &mix);
int run_channel_delta(Stream &st, int run, const LayerWeights &w, const MixerSpec &mix);
int run_experts(Stream &st, const LayerWeights &w, const MlpSpec &mlp);

}  // namespace mynn
