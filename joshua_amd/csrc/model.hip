// Models behind the C ABI: loading by architecture, steps, the greedy pick, and the four plugin symbols
// (declared in include/joshua_hip.h).
#include "model.hpp"

#include <sys/stat.h>

#include "gguf.hpp"
#include "json.hpp"
#include "kernels_graph.hpp"

jq_model::~jq_model() {
    for (void *p : {(void *)logits, (void *)pick, (void *)pick_v, (void *)pick_i})
        if (p) (void)hipFree(p);
}

int jq_model::init_outputs() {
    if (hipMalloc((void **)&pick, sizeof(uint32_t)) != hipSuccess ||
        hipMalloc((void **)&pick_v, jq::ARGMAX_PARTS * sizeof(float)) != hipSuccess ||
        hipMalloc((void **)&pick_i, jq::ARGMAX_PARTS * sizeof(int)) != hipSuccess || reserve_logits(1))
        return fail("%s: logits allocation failed", arch);
    return 0;
}

int jq_model::reserve_logits(size_t rows) {
    if (rows <= logit_cap) return 0;
    float *fresh = nullptr;
    HIP_TRY(hipMalloc((void **)&fresh, rows * vocab * sizeof(float)));
    if (logits) (void)hipFree(logits);  // (waits for what still runs over it)
    logits = fresh, logit_cap = rows;
    return 0;
}

namespace jqh {

static std::vector<ModelArch> &model_archs() {
    static std::vector<ModelArch> v;
    return v;
}
RegisterModelArch::RegisterModelArch(const ModelArch &a) { model_archs().push_back(a); }

}  // namespace jqh

extern "C" {

int jq_model_load(const char *path, uint32_t n_ctx, uint32_t compute, jq_model **out) {
    if (!path || !out) return fail("jq_model_load: null argument");
    *out = nullptr;
    if (compute != JQ_COMPUTE_DEFAULT && compute != JQ_COMPUTE_F32) return fail("jq_model_load: unknown compute format %u", compute);
    struct stat st;
    if (stat(path, &st) != 0) return fail("jq_model_load: no such file or folder: %s", path);
    const bool folder = S_ISDIR(st.st_mode);
    std::string name, err;
    if (folder) {
        jq::Json cfg;
        if (!jq::json_read_file(std::string(path) + "/config.json", &cfg, &err)) return fail("%s", err.c_str());
        const jq::Json *a = cfg.find("architecture");
        if (!a || a->kind != jq::Json::STRING) return fail("config.json: no \"architecture\" in %s", path);
        name = a->str;
    } else {
        auto g = jq::gguf_open(path, &err);
        if (!g) return fail("%s", err.c_str());
        const std::string *a = g->meta_str("general.architecture");
        if (!a) return fail("GGUF: no general.architecture in %s", path);
        name = *a;
    }
    std::string known;
    for (const ModelArch &a : model_archs()) {
        if (a.folder != folder) continue;
        if (name == a.name) return a.load(path, ModelLoadOptions{n_ctx, compute}, out);
        known += std::string(known.empty() ? "`" : ", `") + a.name + "`";
    }
    return fail("no model of architecture `%s`: expected %s", name.c_str(), known.empty() ? "none of this kind" : known.c_str());
}

void jq_model_free(jq_model *m) { delete m; }
uint32_t jq_model_vocab(const jq_model *m) { return m ? m->vocab : 0; }
uint32_t jq_model_context(const jq_model *m) { return m ? m->n_ctx : 0; }
uint32_t jq_model_cached_tokens(const jq_model *m) { return m ? m->n_past : 0; }

int jq_model_forward(jq_model *m, const uint32_t *tokens, uint32_t n_tokens, uint32_t pos, const uint32_t *want,
                     uint32_t n_want, float *logits, int logits_on_device, void *stream) {
    if (!m || !tokens) return fail("jq_model_forward: null argument");
    if (n_want && !want) return fail("jq_model_forward: want is null");
    if (n_tokens == 0) return fail("%s: forward needs at least one token", m->arch);
    std::lock_guard<std::mutex> lock(m->mu);
    // the KV-cache contract of the plugin boundary (reference: crates/joshua-mock-npu/src/lib.rs:89-95)
    if (pos != m->n_past) return fail("%s: pos %u does not match the %u tokens fed so far", m->arch, pos, m->n_past);
    if ((uint64_t)pos + n_tokens > m->n_ctx)
        return fail("%s: %u + %u tokens exceed the context of %u", m->arch, pos, n_tokens, m->n_ctx);
    for (uint32_t i = 0; i < n_tokens; i++)
        if (tokens[i] >= m->vocab) return fail("embedding id %u is out of range for %u rows", tokens[i], m->vocab);
    for (uint32_t i = 0; i < n_want; i++)
        if (want[i] >= n_tokens) return fail("%s: logits wanted at place %u of %u tokens", m->arch, want[i], n_tokens);
    hipStream_t s = (hipStream_t)stream;
    if (m->reserve_logits(std::max<uint32_t>(n_want, 1))) return 1;
    if (m->step(tokens, n_tokens, want, n_want, s)) return 1;
    m->n_past = pos + n_tokens;
    m->logit_rows = n_want;
    if (logits && n_want) {
        HIP_TRY(hipMemcpyAsync(logits, m->logits, (size_t)n_want * m->vocab * sizeof(float),
                               logits_on_device ? hipMemcpyDeviceToDevice : hipMemcpyDeviceToHost, s));
        if (!logits_on_device) HIP_TRY(hipStreamSynchronize(s));
    }
    return 0;
}

int jq_model_greedy(jq_model *m, uint32_t *token, void *stream) {
    if (!m || !token) return fail("jq_model_greedy: null argument");
    hipStream_t s = (hipStream_t)stream;
    std::lock_guard<std::mutex> lock(m->mu);
    const float *row = m->logits + (m->logit_rows > 1 ? m->logit_rows - 1 : 0) * (size_t)m->vocab;
    hipLaunchKernelGGL(jq::argmax_last_parts, dim3(jq::ARGMAX_PARTS), dim3(256), 0, s, row, (int)m->vocab,
                       m->pick_v, m->pick_i);
    hipLaunchKernelGGL(jq::argmax_last_merge, dim3(1), dim3(jq::ARGMAX_PARTS), 0, s, m->pick_v, m->pick_i, m->pick);
    HIP_TRY(hipMemcpyAsync(token, m->pick, sizeof(uint32_t), hipMemcpyDeviceToHost, s));
    HIP_TRY(hipStreamSynchronize(s));
    return 0;
}

int jq_model_reset(jq_model *m) {
    if (!m) return fail("jq_model_reset: model is null");
    std::lock_guard<std::mutex> lock(m->mu);
    m->n_past = 0;
    m->forget();
    return 0;
}

// The four symbols the reference engine binds when it loads a backend as a shared library
// (reference: src/npu/mod.rs:32-50 contract, src/npu/vendor.rs:17-20 signatures, :49-56 symbol
// check, :95-121 init; crates/joshua-mock-npu/src/lib.rs:41-131 return codes of the model plugin).
int32_t joshua_npu_init(const char *model_path, uint32_t n_ctx, uint32_t *out_vocab, void **out_handle) {
    if (!model_path || !out_vocab || !out_handle) return -1;
    *out_handle = nullptr;
    jq_model *m = nullptr;
    if (jq_model_load(model_path, n_ctx, JQ_COMPUTE_DEFAULT, &m)) return -2;
    *out_vocab = m->vocab;
    *out_handle = m;
    return 0;
}

int32_t joshua_npu_forward(void *handle, const uint32_t *tokens, uint32_t n_tokens, uint32_t pos, float *out_logits) {
    if (!handle || !tokens || !out_logits || n_tokens == 0) return -1;
    jq_model *m = (jq_model *)handle;
    // the handle may arrive on another thread than the one that made it; the device is per thread
    if (hipSetDevice(current_device_index()) != hipSuccess) return -5;
    {
        std::lock_guard<std::mutex> lock(m->mu);
        if (pos != m->n_past) return -3;
        if ((uint64_t)pos + n_tokens > m->n_ctx) return -4;
    }
    const uint32_t last = n_tokens - 1;
    return jq_model_forward(m, tokens, n_tokens, pos, &last, 1, out_logits, 0, nullptr) ? -5 : 0;
}

int32_t joshua_npu_reset(void *handle) {
    if (!handle) return -1;
    return jq_model_reset((jq_model *)handle) ? -5 : 0;
}

void joshua_npu_free(void *handle) {
    if (!handle) return;
    (void)hipSetDevice(current_device_index());
    jq_model_free((jq_model *)handle);
}

}  // extern "C"
