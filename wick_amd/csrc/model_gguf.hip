// GGUF files behind the model handle of include/wick_rocm_model.h: the LFM2 handle as one more model class, and the loader that
// looks at a path.  Host code only.
#include <sys/stat.h>

#include <cstring>

#include "../../include/wick_gguf.h"
#include "../../include/wick_rocm_lfm2.h"
#include "../../include/wick_safetensors.h"
#include "model.h"

namespace {

struct Lfm2Adapter final : wick_rocm_model {
    wick_rocm_lfm2* m = nullptr;

    void release(wick_rocm_ctx* ctx) override { wick_rocm_lfm2_free(ctx, m); }
    size_t memory_bytes() const override { return wick_rocm_lfm2_gpu_memory_bytes(m); }
    void set_graph_replay(bool on) override { wick_rocm_lfm2_set_graph_replay(m, on); }
    int reset(wick_rocm_ctx* ctx) override { return wick_rocm_lfm2_reset(ctx, m); }
    int forward(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos, const uint32_t* want, uint32_t n_want, float* logits,
                float* layers) override {
        if (layers) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model: lfm2 keeps no per-layer copies");
        if (pos == 0)
            if (int rc = wick_rocm_lfm2_reset(ctx, m)) return rc;
        uint32_t done = 0;
        for (uint32_t i = 0; i < n_want; i++) {  // a prompt pass returns its last token's logits: one pass per wanted token
            if (int rc = wick_rocm_lfm2_forward_prefill(ctx, m, tokens + done, want[i] + 1 - done, pos + done, logits + (size_t)i * info.vocab_size)) return rc;
            done = want[i] + 1;
        }
        return done < n ? wick_rocm_lfm2_forward_prefill(ctx, m, tokens + done, n - done, pos + done, nullptr) : WICK_ROCM_OK;
    }
    int generate(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out) override {
        if (pos == 0)
            if (int rc = wick_rocm_lfm2_reset(ctx, m)) return rc;
        return wick_rocm_lfm2_generate_greedy(ctx, m, token, pos, n, out);
    }
    size_t state_bytes(uint32_t seq_len) const override { return wick_rocm_lfm2_state_bytes(m, seq_len); }
    int snapshot(wick_rocm_ctx* ctx, uint32_t seq_len, void* out) override { return wick_rocm_lfm2_snapshot_state(ctx, m, seq_len, out, state_bytes(seq_len)); }
    int restore(wick_rocm_ctx* ctx, uint32_t seq_len, const void* in) override { return wick_rocm_lfm2_restore_state(ctx, m, seq_len, in, state_bytes(seq_len)); }
};

int ctx_fail(wick_rocm_ctx* ctx, int code, const std::string& what) {
    std::lock_guard<std::recursive_mutex> lk(ctx->mu);
    return fail(ctx, code, what.c_str());
}

}  // namespace

extern "C" {

int wick_rocm_model_from_gguf(wick_rocm_ctx* ctx, const wick_gguf* gguf, int dtype, uint32_t context_size, wick_rocm_model** out) {
    if (!ctx) return WICK_ROCM_ERR_INVALID_ARG;
    if (!gguf || !out) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_gguf: null argument");
    *out = nullptr;
    if (dtype != WICK_ROCM_MODEL_NATIVE)
        return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_gguf: block-quantized models run on their own types only");
    const char* arch = nullptr;
    size_t len = 0;
    if (wick_gguf_get_str(gguf, "general.architecture", &arch, &len) != 0 || std::string(arch, len) != "lfm2")
        return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_from_gguf: general.architecture is not lfm2");
    wick_rocm_lfm2* m = nullptr;
    if (int rc = wick_rocm_lfm2_load(ctx, gguf, context_size, &m)) return rc;
    wick_rocm_lfm2_config c;
    wick_rocm_lfm2_get_config(m, &c);
    Lfm2Adapter* a = new Lfm2Adapter;
    a->m = m;
    strcpy(a->info.architecture, "lfm2");
    a->info.vocab_size = c.vocab_size, a->info.hidden_size = c.hidden_size, a->info.max_seq_len = c.max_seq_len;
    a->info.layer_runs = c.n_layers, a->info.dtype = dtype;
    *out = a;
    return WICK_ROCM_OK;
}

int wick_rocm_model_load(wick_rocm_ctx* ctx, const char* path, int dtype, uint32_t context_size, wick_rocm_model** out) {
    if (!ctx) return WICK_ROCM_ERR_INVALID_ARG;
    if (!path || !out) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "model_load: null argument");
    *out = nullptr;
    struct stat sb;
    if (stat(path, &sb) != 0) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, std::string("model_load: no such path: ") + path);
    if (S_ISDIR(sb.st_mode)) {
        wick_safetensors* s = nullptr;
        if (wick_safetensors_open(path, &s) != 0) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, std::string("model_load: ") + wick_safetensors_last_error());
        const int rc = wick_rocm_model_from_folder(ctx, s, dtype, context_size, out);
        wick_safetensors_close(s);
        return rc;
    }
    wick_gguf* g = nullptr;
    if (wick_gguf_open(path, &g) != 0) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, std::string("model_load: ") + wick_gguf_last_error());
    const int rc = wick_rocm_model_from_gguf(ctx, g, dtype, context_size, out);
    wick_gguf_close(g);
    return rc;
}

}  // extern "C"
