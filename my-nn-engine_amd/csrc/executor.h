// The executor's state, shared by the model families it runs (decoder.hip: the Llama graph; layered.hip: decoders
// described layer by layer) and by the step machinery around them: inputs, graph capture, loop, profile.
#pragma once
#include <cstring>
#include <map>
#include <mutex>
#include <vector>

#include "attention.h"
#include "kernels.h"
#include "kv_pages.h"

namespace mynn {

struct Lin {
    const void *w = nullptr;      // int8 [N,K] when scale != nullptr, else T [N,K]
    const void *scale = nullptr;  // T [N]
    int N = 0, K = 0;
};

struct Layer {
    const void *norm1 = nullptr, *norm2 = nullptr;
    Lin qkv, o, gate, up, gu, down;  // qkv = rows of q,k,v concatenated; gu = gate/up rows interleaved
    void *k_cache = nullptr, *v_cache = nullptr;
    void *k_scale = nullptr, *v_scale = nullptr;  // int8 KV cache: per-token scales [B,Hkv,max_seq]
    // (everything below points into the model's WeightSet)
    void *qkv_b = nullptr;  // qkv_bias: the q, k, v projection biases concatenated [QD + 2 KD], T
    // prefill executors: weights dequantised once to the 16-bit type, [N, Kp] (wt_gu: gate/up in groups of 32)
    void *wt_qkv = nullptr, *wt_o = nullptr, *wt_gu = nullptr, *wt_down = nullptr;
    // few-row executors: int8 weights re-tiled so that a wave streams them sequentially
    void *pk_qkv = nullptr, *pk_o = nullptr, *pk_gu = nullptr, *pk_down = nullptr;
    // W8A8 prefill executors: int8 gate/up rows and their scales interleaved in groups of 32 (SwiGLU store)
    void *q8_gu = nullptr, *q8_gu_scale = nullptr;
};

// Every copy the library derives from a checkpoint's weights, made at most once and shared by the executors of a
// session (prefill, decode, few-row): the q|k|v and gate/up repacks, the 16-bit resident copy of the matrix-core path,
// the tiled int8 copy of the few-row path, the W8A8 gate/up interleave.  A copy is made by the first executor that
// needs it (under the set's mutex) and lives until the last holder -- the caller's handle or a model -- lets go.
struct WeightLayer {
    void *qkv_w = nullptr, *qkv_s = nullptr, *gu_w = nullptr, *gu_s = nullptr, *qkv_b = nullptr;
    void *wt_qkv = nullptr, *wt_o = nullptr, *wt_gu = nullptr, *wt_down = nullptr;
    void *pk_qkv = nullptr, *pk_o = nullptr, *pk_gu = nullptr, *pk_down = nullptr;
    void *q8_gu = nullptr, *q8_gu_scale = nullptr;
};
struct LayeredWeights;  // the padded copies of a layered model (layered.hip)
void layered_weights_free(LayeredWeights *w);
struct WeightSet {
    std::mutex mu;
    int refs = 1;
    // what the copies depend on: the shapes, the storage type, the caller's buffers
    int n_layers = 0, hidden = 0, n_heads = 0, n_kv_heads = 0, head_dim = 0, ffn = 0, vocab = 0, dtype = 0, int8_weights = 0, qkv_bias = 0, arch = 0;
    LayeredWeights *layered = nullptr;
    std::vector<void *> initializer;
    std::vector<WeightLayer> layers;
    void *wt_lm_head = nullptr, *pk_lm_head = nullptr;
    bool repacked = false, resident16 = false, packed8 = false, q8 = false;
    size_t bytes_repack = 0, bytes_resident16 = 0, bytes_packed8 = 0, bytes_q8 = 0;
};
struct Launch {
    const char *name;
    double bytes;
    double flops;
};

struct LayeredNet;  // layered.hip: what a model described layer by layer has beyond the fields below
struct Model {
    mynn_model_config cfg{};
    LayeredNet *net = nullptr;  // null: the Llama graph
    // the step in flight: new tokens per sequence (the Llama graph: always seq_q), and the rows whose logits it makes,
    // sel_first + i * sel_stride of the batch * rows_now rows (the Llama graph: all)
    int rows_now = 0, sel_first = 0, sel_stride = 1, sel_count = 0;
    int logits_dtype = 0;
    bool quant = true;
    Lin embed, lm_head;
    const void *final_norm = nullptr;
    std::vector<Layer> layers;
    void *wt_lm_head = nullptr, *pk_lm_head = nullptr;
    WeightSet *wset = nullptr;  // the derived weight copies (shared with the session's other executors)
    bool w8a8_fused = false;  // W8A8 with the large int8 tiles: norm+quantise, residual and SwiGLU ride on the launches
    bool qgemv1 = false;      // W8A8 at batch 1: norm, quantiser, int8 GEMV and residual / SwiGLU of a linear in one launch
    bool resident16 = false;  // the wt_* copies exist and the matrix-core path with fused stores is used
    bool skinny = false;      // 16..64 rows: int8 weights streamed once through the few-row matrix-core kernel
    float *skinny_scratch = nullptr;
    void *cos_t = nullptr, *sin_t = nullptr;
    // arena
    char *arena = nullptr;
    size_t arena_bytes = 0;
    void *x = nullptr, *x2 = nullptr, *nrm = nullptr, *qkv = nullptr, *q = nullptr, *attn = nullptr, *g = nullptr,
         *u = nullptr, *hmid = nullptr, *proj = nullptr, *logits = nullptr;
    int8_t *a8 = nullptr;    // W8A8: the current linear's activation rows as int8 [rows, max(H, QD, F)]
    void *a8_scale = nullptr;  // and their per-row scales [rows]
    int64_t *d_ids = nullptr, *d_pos = nullptr;
    int32_t *d_past = nullptr, *d_active = nullptr, *d_next = nullptr, *d_tokens = nullptr, *d_step = nullptr;
    void *attn_scratch = nullptr;
    int nsplit = 1, slice = 0, heads_per_wg = 1;
    int token_cap = 0;
    // host staging (pinned)
    char *h_stage = nullptr;
    size_t stage_bytes = 0, next_stage = 256;
    hipStream_t stream = nullptr;
    hipGraph_t graph = nullptr;
    hipGraphExec_t graph_exec = nullptr;
    bool use_graph = false;
    int launches = 0;
    // batch-1 decode: projection and attention share a launch; m.qkv is then the hand-over vector between them
    // (all 0xFFFF between uses) and d_past[3] the error word of its bounded waits
    // the device-resident loop replays kLoopSteps steps per graph launch where it can (a graph launch costs the device a
    // few microseconds of its own, a tenth of a batch-1 step's launches)
    hipGraph_t graph_loop = nullptr;
    hipGraphExec_t graph_loop_exec = nullptr;
    bool qkv_attn = false;
    bool lm_argmax = false;       // ... and the lm_head launch finds the greedy token and moves the loop state on
    uint64_t *lm_cand = nullptr;  // its candidate words (all ~0 between launches)
    int spin_limit = 400000;      // polls a consumer role makes before it gives up and raises the error word
    int handover_failures = 0;    // steps whose hand-over gave up; the executor then rebuilt itself with one op per launch
    // what build() had chosen before a give-up switched the shared launches off, and when they are tried again: after
    // rearm_after clean steps (doubled by every further give-up; 0 = never)
    bool shared_qkv_attn = false, shared_lm_argmax = false, fell_back = false;
    int rearm_after = 256;
    long clean_steps = 0;
    // streaming_kv: the ring inputs of the step in flight (host copies: the operators take them at launch time, as the
    // reference's kernels do), kv_position on the device, and the operators' [heads, S, D] tensors
    int ring_sink = 0, ring_window = 0, ring_start = 0, h_past = 0, h_active = 0;
    int64_t *d_kvpos = nullptr;
    void *q_ref = nullptr, *k_new = nullptr, *v_new = nullptr, *attn_ref = nullptr, *k_rot = nullptr;
    void *ring_ws = nullptr;      // ... and the scratch memory of the ring attention (rank-ordered rows, partial results)
    size_t ring_ws_bytes = 0;
    int last_status = 0;          // of the last model() call on this state
    void *warena = nullptr;       // weight_arena: every linear weight and scale of the model in one allocation, in execution order
    mynn_kv_pages *pages = nullptr;  // kv_page_rows: the session's page table (the caller's); k_cache / v_cache then are pools
    KvPaging paging;
    void *ws = nullptr;           // executors that dequantise a weight per call (M >= 16, no resident copy): their own workspace
    // per-launch record of the last enqueue (names + algorithmic bytes), events when profiling
    std::vector<Launch> record;
    bool profiling = false;
    std::vector<hipEvent_t> events;
};

inline size_t align_up(size_t v, size_t a) { return (v + a - 1) / a * a; }

struct ArenaPlan {
    size_t off = 0;
    size_t take(size_t bytes) {
        size_t o = off;
        off = align_up(off + bytes, 256);
        return o;
    }
};

inline void note(Model &m, const char *name, double bytes, double flops = 0.0) {
    if (m.profiling) {
        // the launch that follows stamps these two with its own start and end
        hipEvent_t a, b;
        hipEventCreate(&a);
        hipEventCreate(&b);
        m.events.push_back(a);
        m.events.push_back(b);
        launch_timer() = LaunchTimer{a, b};
    }
    m.record.push_back({name, bytes, flops});
}

#define TRY(expr)            \
    do {                     \
        int rc__ = (expr);   \
        if (rc__) return rc__; \
    } while (0)

// ---- layered.hip
int build_layered(Model &m, void **state);
int enqueue_layered(Model &m);
void destroy_layered(Model &m);

// ---- decoder.hip: a model that takes any number of new tokens up to seq_q in a step (a Llama graph of seq_q > 1 takes
// exactly seq_q; shorter portions are padded and their last rows written over by the next tokens)
bool model_takes_any_rows(const void *state);
// ---- layered.hip: models whose session state stands for all tokens read so far; a copy of it and back (on the model's stream)
bool model_has_sequence_state(const void *state);
int executor_save_state(void *state);
int executor_restore_state(void *state);
int executor_bind_pages(Model &m);

}  // namespace mynn
