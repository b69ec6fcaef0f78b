// One checkpoint on the device and the sessions it serves: config.json through the model registry, weights uploaded once,
// one weight set, and per session a decode executor and a prompt executor over a cache of its own.  Layered models (and
// Llama shapes that have a paged form) take their cache rows from one pool of pages, so sessions of different lengths share
// the memory and a session that ends gives its pages to the next; its sequence states go to the next session the same way.
// Host code; the executors do the rest.
#include <algorithm>
#include <memory>
#include <vector>

#include "executor.h"
#include "model_spec.h"
#include "session.h"

using namespace mynn;

struct mynn_engine {
    mynn_engine_options opt{};
    int arch = 0;
    mynn_model_config cfg{};           // decode configuration: seq_q 1, batch 1
    mynn_device_weights *weights = nullptr;
    mynn_weight_set *set = nullptr;
    mynn_kv_pool *pool = nullptr;      // null: a session owns contiguous caches
    std::vector<void *> pool_buffers;
    std::vector<std::vector<void *>> slots;  // sequence states of ended sessions (one buffer per state), for the next ones
    int sessions = 0;
    int prefill_rows = 0;
};

namespace {
struct EngineSession {
    mynn_engine *engine;
    mynn_kv_pages *pages = nullptr;
    std::vector<void *> caches;  // contiguous caches (no pool)
    std::vector<void *> slot;    // sequence states
};

// the session-state buffers with a row per token (PER_TOKEN) or a block per sequence; null where the other kind belongs
enum StateKind { PER_TOKEN, PER_SEQUENCE };
int state_buffers(const mynn_engine &e, StateKind kind, size_t rows, std::vector<void *> &out) {
    const int n = mynn_arch_state_count(e.arch);
    for (int i = 0; i < n; i++) {
        void *p = nullptr;
        const size_t bytes = kind == PER_TOKEN ? rows * mynn_arch_state_row_bytes(e.arch, i, e.opt.dtype) : mynn_arch_state_seq_bytes(e.arch, i);
        if (bytes) MYNN_HIP(hipMalloc(&p, bytes));
        out.push_back(p);
        if (bytes) MYNN_HIP(hipMemset(p, 0, bytes));
    }
    return 0;
}

int open_engine(mynn_engine &e, const char *dir, const mynn_engine_options &opt) {
    e.opt = opt;
    if (e.opt.max_seq <= 0) e.opt.max_seq = e.opt.max_tokens;
    if (e.opt.prefill_rows <= 0) e.opt.prefill_rows = 512;
    if (e.opt.page_rows <= 0) e.opt.page_rows = 64;
    MYNN_REQUIRE(e.opt.max_tokens > 0 && e.opt.max_seq > 0, MYNN_ERR_INVALID, "engine: max_tokens %d, max_seq %d", opt.max_tokens, opt.max_seq);
    const int P = e.opt.page_rows, max_seq = (e.opt.max_seq + P - 1) / P * P;
    e.opt.max_seq = max_seq;
    e.prefill_rows = std::min(e.opt.prefill_rows, max_seq);
    e.arch = mynn_arch_open(dir);
    if (e.arch < 0) return e.arch;
    int rc = mynn_arch_config(e.arch, e.opt.dtype, max_seq, 1, 1, &e.cfg);
    if (rc) return rc;
    const bool layered = e.cfg.arch != 0;
    const bool paged = layered || (attn_stream_paged_supported(1, e.cfg.n_heads, e.cfg.n_kv_heads, e.cfg.head_dim, e.opt.dtype, P) && max_seq / P <= 64);
    if (paged) e.cfg.kv_page_rows = P;
    mynn_weights *w = mynn_weights_open(dir);
    if (!w) return MYNN_ERR_INVALID;
    e.weights = mynn_weights_upload(w, &e.cfg);
    mynn_weights_close(w);
    if (!e.weights) return MYNN_ERR_INVALID;
    e.cfg.weights_int8 = mynn_device_weights_int8(e.weights);
    e.set = mynn_weight_set_create(&e.cfg, mynn_device_weights_initializer(e.weights));
    if (!e.set) return MYNN_ERR_INVALID;
    if (paged) {
        const int n_pages = (e.opt.max_tokens + P - 1) / P + 8;  // (a session's last page is rarely full)
        e.pool = mynn_kv_pool_create(n_pages, P);
        if (!e.pool) return MYNN_ERR_INVALID;
        rc = state_buffers(e, PER_TOKEN, (size_t)n_pages * P, e.pool_buffers);
    }
    return rc;
}

void release_session(mynn_llm *l) {
    EngineSession *s = (EngineSession *)l->owner;
    if (l->prefill) model_destroy(l->prefill);
    if (l->decode) model_destroy(l->decode);
    if (s->pages) (void)mynn_kv_pages_destroy(s->pages);
    for (void *p : s->caches) (void)hipFree(p);
    if (!s->slot.empty()) s->engine->slots.push_back(std::move(s->slot));
    s->engine->sessions--;
    delete s;
}
}  // namespace

extern "C" int mynn_engine_close(mynn_engine *e) {
    if (!e) return 0;
    MYNN_REQUIRE(e->sessions == 0, MYNN_ERR_STATE, "engine_close: %d sessions live", e->sessions);
    if (e->set) mynn_weight_set_destroy(e->set);
    if (e->weights) mynn_device_weights_free(e->weights);
    if (e->pool) (void)mynn_kv_pool_destroy(e->pool);
    for (void *p : e->pool_buffers) (void)hipFree(p);
    for (auto &slot : e->slots)
        for (void *p : slot) (void)hipFree(p);
    delete e;
    return 0;
}

extern "C" mynn_engine *mynn_engine_open(const char *model_dir, const mynn_engine_options *opt) {
    if (!model_dir || !opt) {
        fail(MYNN_ERR_INVALID, "engine_open: null argument");
        return nullptr;
    }
    mynn_engine *e = new mynn_engine;
    if (open_engine(*e, model_dir, *opt)) {
        (void)mynn_engine_close(e);
        return nullptr;
    }
    return e;
}

extern "C" int mynn_engine_vocab(const mynn_engine *e) { return e ? e->cfg.vocab : MYNN_ERR_INVALID; }
extern "C" int mynn_engine_free_rows(mynn_engine *e) {
    return e && e->pool ? mynn_kv_pool_free_pages(e->pool) * e->opt.page_rows : -1;
}

extern "C" mynn_llm *mynn_engine_session(mynn_engine *e, int64_t eos_token_id) {
    if (!e) {
        fail(MYNN_ERR_INVALID, "engine_session: null engine");
        return nullptr;
    }
    auto *s = new EngineSession{e};
    auto *l = new mynn_llm;
    l->owner = s;
    l->release = release_session;
    e->sessions++;
    std::vector<void *> state = e->pool_buffers;
    bool ok = true;
    if (e->slots.empty()) ok = state_buffers(*e, PER_SEQUENCE, 1, s->slot) == 0;
    else {
        s->slot = std::move(e->slots.back());
        e->slots.pop_back();
    }
    if (ok && !e->pool) {
        ok = state_buffers(*e, PER_TOKEN, e->opt.max_seq, s->caches) == 0;
        state = s->caches;
    }
    for (size_t i = 0; ok && i < state.size(); i++)
        if (s->slot[i]) state[i] = s->slot[i];
    if (ok && e->pool) {
        s->pages = mynn_kv_pages_create(e->pool, 1, e->opt.max_seq);
        ok = s->pages != nullptr;
        state.push_back(s->pages);
    }
    mynn_model_config cfg = e->cfg;
    if (ok) l->decode = mynn_model_create_shared(&cfg, e->set, state.data());
    cfg.seq_q = e->prefill_rows;
    if (l->decode && cfg.seq_q > 1) l->prefill = mynn_model_create_shared(&cfg, e->set, state.data());
    if (!l->decode || (cfg.seq_q > 1 && !l->prefill)) {
        mynn_llm_destroy(l);
        return nullptr;
    }
    l->prefill_len = l->prefill ? cfg.seq_q : 0;
    l->max_seq = e->opt.max_seq;
    l->eos = eos_token_id;
    l->seq_state = model_has_sequence_state(l->decode);
    return l;
}
