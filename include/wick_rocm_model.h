/* wick_rocm_model.h -- one handle over every model the library knows, chosen by what the file says it is.
 *
 * A model folder (config.json + model.safetensors, include/wick_safetensors.h) is loaded as the architecture its config.json names;
 * a GGUF file as the one its general.architecture names.  Both come back as the same handle with the step calls of the reference's
 * `trait Model` (wick/src/model/mod.rs:72-323): prompts, single steps, greedy generation, state snapshots.  Same context, status
 * codes and locking as include/wick_rocm.h.
 *
 * The handle holds ONE sequence's state and no position of its own: `pos` / `start_pos` are the caller's, and a call at position 0
 * starts a new sequence.  Several sequences take turns through snapshots.
 */
#ifndef WICK_ROCM_MODEL_H
#define WICK_ROCM_MODEL_H

#include "wick_rocm.h"

#ifdef __cplusplus
extern "C" {
#endif

struct wick_gguf;
struct wick_safetensors;
typedef struct wick_rocm_model wick_rocm_model;

/* What a model computes in.  WICK_ROCM_MODEL_NATIVE: the types it is served with (a model folder: bfloat16 matrix products with f32
 * accumulation, f32 norms / attention weights / recurrences / residual; GGUF: its block types, f32 KV rows).  WICK_ROCM_MODEL_F32:
 * f32 activations, caches and products throughout (model folders; the bfloat16 weights are widened exactly). */
enum { WICK_ROCM_MODEL_NATIVE = 0, WICK_ROCM_MODEL_F32 = 1 };

typedef struct wick_rocm_model_info {
    char architecture[32];
    uint32_t vocab_size, hidden_size, max_seq_len;
    uint32_t layer_runs; /* layers a token goes through (a looped layer counts every time) */
    int dtype;
} wick_rocm_model_info;

/* The architectures model folders may name, in the order of the registry; null behind the last one. */
const char *wick_rocm_model_folder_architecture(uint32_t index);

int wick_rocm_model_from_folder(wick_rocm_ctx *ctx, const struct wick_safetensors *folder, int dtype, uint32_t context_size, wick_rocm_model **out);
int wick_rocm_model_from_gguf(wick_rocm_ctx *ctx, const struct wick_gguf *gguf, int dtype, uint32_t context_size, wick_rocm_model **out);
/* Opens `path` (a model folder, or a GGUF file) and loads it. */
int wick_rocm_model_load(wick_rocm_ctx *ctx, const char *path, int dtype, uint32_t context_size, wick_rocm_model **out);
int wick_rocm_model_free(wick_rocm_ctx *ctx, wick_rocm_model *model);
int wick_rocm_model_get_info(const wick_rocm_model *model, wick_rocm_model_info *out);
/* Model::gpu_memory_bytes. */
size_t wick_rocm_model_gpu_memory_bytes(const wick_rocm_model *model);
/* Steps replay a captured graph; 0 enqueues the same launches one by one (per-dispatch timing, kernel tracers). */
int wick_rocm_model_set_graph_replay(wick_rocm_model *model, int enabled);
int wick_rocm_model_reset(wick_rocm_ctx *ctx, wick_rocm_model *model);

/* n tokens at positions start_pos .. start_pos + n - 1; logits [n_want][vocab_size] of the tokens want[0] < want[1] < .. (indices
 * among these n; may be none).  One or two tokens run as single steps, more as prompt passes. */
int wick_rocm_model_forward(wick_rocm_ctx *ctx, wick_rocm_model *model, const uint32_t *tokens, uint32_t n, uint32_t start_pos,
                            const uint32_t *want, uint32_t n_want, float *logits);
/* The same as one prompt pass that also copies out the residual stream after every layer run, layers [layer_runs][n][hidden_size]
 * (n at most one pass; a debugging aid, model folders only). */
int wick_rocm_model_forward_layers(wick_rocm_ctx *ctx, wick_rocm_model *model, const uint32_t *tokens, uint32_t n, uint32_t start_pos, float *layers);
/* Model::forward_prefill_chunked (wick/src/model/mod.rs:111-140) over wick_rocm_model_forward: chunks of `ubatch` tokens (0 = one
 * chunk), `cancel` (may be null) read after every chunk, *consumed = tokens that made it into the state, logits of the last one. */
int wick_rocm_model_prefill_chunked(wick_rocm_ctx *ctx, wick_rocm_model *model, const uint32_t *tokens, uint32_t n, uint32_t start_pos,
                                    uint32_t ubatch, const volatile int32_t *cancel, uint32_t *consumed, float *logits);
/* n greedy steps starting with `token` at `pos`, picks on the device: out_tokens[i] is the pick after step i. */
int wick_rocm_model_generate_greedy(wick_rocm_ctx *ctx, wick_rocm_model *model, uint32_t token, uint32_t pos, uint32_t n, uint32_t *out_tokens);

/* Model::snapshot_state / restore_state: the state after seq_len positions as host bytes. */
size_t wick_rocm_model_state_bytes(const wick_rocm_model *model, uint32_t seq_len);
int wick_rocm_model_snapshot_state(wick_rocm_ctx *ctx, wick_rocm_model *model, uint32_t seq_len, void *out, size_t nbytes);
int wick_rocm_model_restore_state(wick_rocm_ctx *ctx, wick_rocm_model *model, uint32_t seq_len, const void *in, size_t nbytes);

#ifdef __cplusplus
}
#endif
#endif /* WICK_ROCM_MODEL_H */
