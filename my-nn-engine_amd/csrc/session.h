// LlmSession (crates/llm/src/session.rs:311-537): the state behind mynn_llm.
#pragma once
#include "mynn_common.h"

struct mynn_llm {
    void *decode = nullptr, *prefill = nullptr;
    int prefill_len = 0, max_seq = 0;
    int64_t eos = -1, past_len = 0;
    mynn_step_fn step = nullptr;
    void *user = nullptr;
    int last_error = 0;
    void (*release)(mynn_llm *) = nullptr;  // an engine's session: gives its executors and cache back
    void *owner = nullptr;
    // models with a sequence state (recurrences): it stands for the first state_len tokens, and only they can be continued
    bool seq_state = false;
    int64_t state_len = 0;
    bool streaming = false;  // DecodeKind::LlamaStreaming { sink, window }
    int sink = 0, window = 0;
};
