// C ABI of include/wick_rocm_model.h over the model interface, and the registry of folder architectures.  Host code only.
#include <cstring>

#include "model.h"
#include "model_folder.h"

namespace {

// The architectures config.json may name.
constexpr FolderModelClass kFolderModels[] = {
    {"Lokinex", load_lokinex},
    {"Zirurax", load_zirurax},
};
constexpr uint32_t kFolderModelCount = sizeof(kFolderModels) / sizeof(kFolderModels[0]);

int ctx_fail(wick_rocm_ctx* ctx, int code, const std::string& what) {
    std::lock_guard<std::recursive_mutex> lk(ctx->mu);
    return fail(ctx, code, what.c_str());
}

int check_tokens(wick_rocm_ctx* ctx, const wick_rocm_model* m, const uint32_t* tokens, uint32_t n, uint32_t pos, uint32_t ahead) {
    for (uint32_t i = 0; i < n; i++)
        if (tokens[i] >= m->info.vocab_size) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: token id out of range");
    if ((uint64_t)pos + ahead > m->info.max_seq_len) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: position beyond the context size");
    return WICK_ROCM_OK;
}

// Nothing else gets onto the context's stream (or into a capture) while a call holds both locks.
struct StepLock {
    std::lock_guard<std::mutex> model;
    std::lock_guard<std::recursive_mutex> ctx;
    StepLock(wick_rocm_ctx* c, wick_rocm_model* m) : model(m->mu), ctx(c->mu) {}
};

}  // namespace

extern "C" {

const char* wick_rocm_model_folder_architecture(uint32_t index) { return index < kFolderModelCount ? kFolderModels[index].architecture : nullptr; }

int wick_rocm_model_from_folder(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out) {
    if (!ctx) return WICK_ROCM_ERR_INVALID_ARG;
    if (!folder || !out) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_folder: null argument");
    *out = nullptr;
    if (dtype != WICK_ROCM_MODEL_NATIVE && dtype != WICK_ROCM_MODEL_F32) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_folder: unknown dtype");
    if (context_size == 0) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_folder: context_size must be > 0");
    for (const FolderModelClass& c : kFolderModels)
        if (folder->architecture == c.architecture) return c.load(ctx, folder, dtype, context_size, out);
    return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_folder: unknown architecture " + folder->architecture);
}

int wick_rocm_model_free(wick_rocm_ctx* ctx, wick_rocm_model* model) {
    if (!ctx) return WICK_ROCM_ERR_INVALID_ARG;
    if (!model) return WICK_ROCM_OK;
    model->release(ctx);
    delete model;
    return WICK_ROCM_OK;
}

int wick_rocm_model_get_info(const wick_rocm_model* model, wick_rocm_model_info* out) {
    if (!model || !out) return WICK_ROCM_ERR_INVALID_ARG;
    *out = model->info;
    return WICK_ROCM_OK;
}

size_t wick_rocm_model_gpu_memory_bytes(const wick_rocm_model* model) { return model ? model->memory_bytes() : 0; }

int wick_rocm_model_set_graph_replay(wick_rocm_model* model, int enabled) {
    if (!model) return WICK_ROCM_ERR_INVALID_ARG;
    std::lock_guard<std::mutex> lk(model->mu);
    model->set_graph_replay(enabled != 0);
    return WICK_ROCM_OK;
}

int wick_rocm_model_reset(wick_rocm_ctx* ctx, wick_rocm_model* model) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    StepLock lk(ctx, model);
    return model->reset(ctx);
}

int wick_rocm_model_forward(wick_rocm_ctx* ctx, wick_rocm_model* model, const uint32_t* tokens, uint32_t n, uint32_t start_pos, const uint32_t* want,
                            uint32_t n_want, float* logits) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    if (!tokens || n == 0) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: no tokens");
    if (n_want && (!want || !logits)) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: null want or logits");
    for (uint32_t i = 0; i < n_want; i++)
        if (want[i] >= n || (i > 0 && want[i] <= want[i - 1])) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: want must ascend below the token count");
    StepLock lk(ctx, model);
    if (int rc = check_tokens(ctx, model, tokens, n, start_pos, n)) return rc;
    return model->forward(ctx, tokens, n, start_pos, want, n_want, logits, nullptr);
}

int wick_rocm_model_forward_layers(wick_rocm_ctx* ctx, wick_rocm_model* model, const uint32_t* tokens, uint32_t n, uint32_t start_pos, float* layers) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    if (!tokens || n == 0 || !layers) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: no tokens or null layers");
    StepLock lk(ctx, model);
    if (int rc = check_tokens(ctx, model, tokens, n, start_pos, n)) return rc;
    return model->forward(ctx, tokens, n, start_pos, nullptr, 0, nullptr, layers);
}

int wick_rocm_model_prefill_chunked(wick_rocm_ctx* ctx, wick_rocm_model* model, const uint32_t* tokens, uint32_t n, uint32_t start_pos, uint32_t ubatch,
                                    const volatile int32_t* cancel, uint32_t* consumed, float* logits) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    if (!consumed) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model prefill: null consumed pointer");
    *consumed = 0;
    if (n == 0) return WICK_ROCM_OK;
    const uint32_t step = ubatch == 0 ? n : ubatch;
    while (*consumed < n) {
        const uint32_t len = n - *consumed < step ? n - *consumed : step, last = len - 1;
        if (int rc = wick_rocm_model_forward(ctx, model, tokens + *consumed, len, start_pos + *consumed, &last, logits ? 1u : 0u, logits)) return rc;
        *consumed += len;
        if (cancel && __atomic_load_n(cancel, __ATOMIC_RELAXED) != 0) break;  // after a chunk: a call always makes progress
    }
    return WICK_ROCM_OK;
}

int wick_rocm_model_generate_greedy(wick_rocm_ctx* ctx, wick_rocm_model* model, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out_tokens) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    if (!out_tokens) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: null output pointer");
    if (n == 0) return WICK_ROCM_OK;
    StepLock lk(ctx, model);
    if (int rc = check_tokens(ctx, model, &token, 1, pos, n)) return rc;
    return model->generate(ctx, token, pos, n, out_tokens);
}

size_t wick_rocm_model_state_bytes(const wick_rocm_model* model, uint32_t seq_len) {
    return model && seq_len <= model->info.max_seq_len ? model->state_bytes(seq_len) : 0;
}

int wick_rocm_model_snapshot_state(wick_rocm_ctx* ctx, wick_rocm_model* model, uint32_t seq_len, void* out, size_t nbytes) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    StepLock lk(ctx, model);
    if (seq_len > model->info.max_seq_len || nbytes != model->state_bytes(seq_len) || (!out && nbytes))
        return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model snapshot: the buffer must hold exactly wick_rocm_model_state_bytes(model, seq_len) bytes");
    return model->snapshot(ctx, seq_len, out);
}

int wick_rocm_model_restore_state(wick_rocm_ctx* ctx, wick_rocm_model* model, uint32_t seq_len, const void* in, size_t nbytes) {
    if (!ctx || !model) return WICK_ROCM_ERR_INVALID_ARG;
    StepLock lk(ctx, model);
    if (seq_len > model->info.max_seq_len || nbytes != model->state_bytes(seq_len) || (!in && nbytes))
        return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model restore: the snapshot must hold exactly wick_rocm_model_state_bytes(model, seq_len) bytes");
    return model->restore(ctx, seq_len, in);
}

}  // extern "C"
