// The interface behind include/wick_rocm_model.h and the registry of model classes.  Not installed.
#pragma once

#include "../../include/wick_rocm_model.h"
#include "wick_rocm_ctx.h"

// Every call arrives with the model's and the context's lock held and its arguments checked against `info`.
struct wick_rocm_model {
    wick_rocm_model_info info{};
    std::mutex mu;

    virtual ~wick_rocm_model() = default;
    // Gives back what the model holds on the device.
    virtual void release(wick_rocm_ctx* ctx) = 0;
    virtual size_t memory_bytes() const = 0;
    virtual void set_graph_replay(bool on) = 0;
    virtual int reset(wick_rocm_ctx* ctx) = 0;
    // layers (null, or [layer_runs][n][hidden_size]): the residual stream after every layer run.
    virtual int forward(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos, const uint32_t* want, uint32_t n_want, float* logits,
                        float* layers) = 0;
    virtual int generate(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out) = 0;
    virtual size_t state_bytes(uint32_t seq_len) const = 0;
    virtual int snapshot(wick_rocm_ctx* ctx, uint32_t seq_len, void* out) = 0;
    virtual int restore(wick_rocm_ctx* ctx, uint32_t seq_len, const void* in) = 0;
};

// A model class for folders: loads the folder or says what is wrong with it (the context's last error).
struct FolderModelClass {
    const char* architecture;
    int (*load)(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out);
};

int load_lokinex(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out);
int load_zirurax(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out);

// One step of a model on the context's stream: a replay of the graph in `slot` (captured when there is none yet, or when the
// context's scratch moved since), or, without `use_graph` or while per-dispatch timing is on, the launches of `enqueue` one by one.
template <typename Enqueue>
inline int run_step_graph(wick_rocm_ctx* ctx, wick_rocm_graph*& slot, bool use_graph, Enqueue&& enqueue) {
    bool timing;
    {
        std::lock_guard<std::recursive_mutex> lk(ctx->mu);
        timing = ctx->timer.enabled;
    }
    if (!use_graph || timing) return enqueue();
    if (slot && graph_is_stale(ctx, slot)) {
        wick_rocm_graph_destroy(ctx, slot);
        slot = nullptr;
    }
    if (!slot) {
        if (int rc = wick_rocm_graph_begin(ctx)) return rc;
        const int rc = enqueue();
        wick_rocm_graph* captured = nullptr;
        const int rc_end = wick_rocm_graph_end(ctx, &captured);  // always end the capture
        if (rc) {
            if (captured) wick_rocm_graph_destroy(ctx, captured);
            return rc;
        }
        if (rc_end) return rc_end;
        slot = captured;
    }
    return wick_rocm_graph_launch(ctx, slot);
}
