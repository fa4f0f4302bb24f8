// A model resident on the device: what every architecture shares (the tokens fed so far, the logits of the last
// step, the greedy pick), and the registry the loader picks an architecture from.
#pragma once
#include "core.hpp"

struct jq_model {
    const char *arch = "";        // for messages
    uint32_t vocab = 0, n_ctx = 0;
    uint32_t n_past = 0;          // tokens fed so far
    float *logits = nullptr;      // [logit_rows][vocab]: the wanted positions of the last step
    size_t logit_cap = 0, logit_rows = 0;
    uint32_t *pick = nullptr;
    float *pick_v = nullptr;      // the greedy pick's candidates, one per slice of the logits
    int *pick_i = nullptr;
    std::mutex mu;

    jq_model() = default;
    jq_model(const jq_model &) = delete;
    jq_model &operator=(const jq_model &) = delete;
    virtual ~jq_model();
    // Enqueues one step: n tokens (host memory) at positions n_past .., and the logits of the `n_want` places among
    // them into `logits` (reserved by the caller), in the order of `want`.
    virtual int step(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, hipStream_t s) = 0;
    // The cached keys, values and recurrent states are those of no sequence from now on.
    virtual void forget() {}
    int init_outputs();           // the pick's buffers and one row of logits
    int reserve_logits(size_t rows);
};

namespace jqh {

struct ModelLoadOptions {
    uint32_t n_ctx;    // tokens the caches hold; 0: what the file says
    uint32_t compute;  // JQ_COMPUTE_*
};

// An architecture by the name its files give: general.architecture of a GGUF file, or "architecture" of the
// config.json in a folder.
struct ModelArch {
    const char *name;
    bool folder;
    int (*load)(const char *path, const ModelLoadOptions &opt, jq_model **out);
};
struct RegisterModelArch {
    explicit RegisterModelArch(const ModelArch &a);
};

}  // namespace jqh
