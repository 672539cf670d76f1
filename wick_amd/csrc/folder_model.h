// What the models of a folder share: reading config.json, packing tensors, and the frame of a model class -- device buffers, steps as
// replayed graphs, prompts cut into passes, wanted logits, snapshots.  A model class fills in its weights, one step and one pass.  Host
// code only, included by the model units.
#pragma once

#include <algorithm>
#include <cmath>
#include <cstring>
#include <map>
#include <memory>
#include <vector>

#include "model.h"
#include "model_folder.h"
#include "wick_rocm_dense.h"

namespace folder_model {

constexpr uint32_t kStepsMax = 2;       // portions this short run as single steps
constexpr uint32_t kHeadRows = 64;      // wanted rows per product with the head
constexpr uint32_t kHeadGemvRows = 4;   // up to this many run as matrix-vector products

enum StepMode { kStepLogits = 0, kStepGreedy = 1, kStepNoHead = 2, kStepModes = 3 };

#define MODEL_LAUNCH(call)                                                  \
    do {                                                                    \
        const hipError_t e_ = (call);                                       \
        if (e_ != hipSuccess) return fail_hip(ctx, e_, "model: " #call);    \
    } while (0)
#define MODEL_TRY(call)                   \
    do {                                  \
        if (int rc_ = (call)) return rc_; \
    } while (0)

// ---- config.json ------------------------------------------------------------------------------------------------------------

struct ConfigError {
    std::string what;
};

inline const Json& need(const Json& j, const char* key, const std::string& where) {
    const Json* v = j.find(key);
    if (!v) throw ConfigError{"config: " + where + " has no \"" + key + "\""};
    return *v;
}
inline double number(const Json& j, const char* key, const std::string& where) {
    const Json& v = need(j, key, where);
    if (v.kind != Json::kNumber || !std::isfinite(v.number)) throw ConfigError{"config: " + where + "." + key + " is not a number"};
    return v.number;
}
inline uint32_t size(const Json& j, const char* key, const std::string& where, uint32_t least = 1) {
    const double v = number(j, key, where);
    if (v < least || v > 1e9 || v != std::floor(v)) throw ConfigError{"config: " + where + "." + key + " is out of range"};
    return (uint32_t)v;
}
inline const std::string& text(const Json& j, const char* key, const std::string& where) {
    const Json& v = need(j, key, where);
    if (v.kind != Json::kString) throw ConfigError{"config: " + where + "." + key + " is not a string"};
    return v.string;
}

// Null and absence read alike.
inline const Json* optional(const Json& j, const char* key) {
    const Json* v = j.find(key);
    return v && !v->is_null() ? v : nullptr;
}

// ---- weights ----------------------------------------------------------------------------------------------------------------

inline float bf16(uint16_t b) {
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

// A bfloat16 tensor of the given shape.
inline const uint16_t* tensor(const wick_safetensors* f, const std::string& name, const std::vector<uint64_t>& shape) {
    const wick_safetensors::Tensor* t = f->find(name);
    if (!t) throw ConfigError{"no tensor " + name};
    if (t->dtype != WICK_SAFETENSORS_BF16 || t->shape != shape) throw ConfigError{"tensor " + name + " has another type or shape than the config says"};
    return reinterpret_cast<const uint16_t*>(t->data);
}
inline float scalar(const wick_safetensors* f, const std::string& name) { return bf16(*tensor(f, name, {})); }

// Host image of a DenseWeight: groups of rows padded to multiples of 64 in both directions.
struct Packer {
    uint32_t mp, kp;
    size_t stride;
    std::vector<uint16_t> v;
    Packer(uint32_t groups, uint32_t rows, uint32_t k) : mp(pad_to(rows, kDensePad)), kp(pad_to(k, kDensePad)), stride((size_t)mp * kp), v(stride * groups, 0) {}
    void row(uint32_t group, uint32_t r, const uint16_t* src, uint32_t n, uint32_t col = 0) {
        memcpy(&v[group * stride + (size_t)r * kp + col], src, (size_t)n * 2);
    }
    void rows(uint32_t group, uint32_t first, const uint16_t* src, uint32_t count, uint32_t n, uint32_t col = 0) {
        for (uint32_t i = 0; i < count; i++) row(group, first + i, src + (size_t)i * n, n, col);
    }
    // Feature f of the first / second of two weights that share a product.
    static uint32_t paired(uint32_t f, bool second) { return f / 16 * 32 + f % 16 + (second ? 16 : 0); }
    void pair(uint32_t group, const uint16_t* first, const uint16_t* second, uint32_t count, uint32_t n, uint32_t col = 0) {
        for (uint32_t i = 0; i < count; i++) {
            row(group, paired(i, false), first + (size_t)i * n, n, col);
            row(group, paired(i, true), second + (size_t)i * n, n, col);
        }
    }
};

inline std::vector<float> widened(const uint16_t* src, size_t n) {
    std::vector<float> v(n);
    for (size_t i = 0; i < n; i++) v[i] = bf16(src[i]);
    return v;
}

// Depthwise taps [channels][taps] as [taps][stride], channel c at at(c).
template <typename At>
std::vector<float> taps_by_time(const uint16_t* w, uint32_t channels, uint32_t taps, uint32_t stride, At&& at) {
    std::vector<float> v((size_t)taps * stride, 0.0f);
    for (uint32_t c = 0; c < channels; c++)
        for (uint32_t k = 0; k < taps; k++) v[(size_t)k * stride + at(c)] = bf16(w[(size_t)c * taps + k]);
    return v;
}

// Cosine and sine of pos * freqs[i], [max_seq][freqs][2], from f64.
inline std::vector<float> rope_table(const std::vector<double>& freqs, uint32_t max_seq) {
    const size_t half = freqs.size();
    std::vector<float> t((size_t)max_seq * half * 2);
    for (size_t j = 0; j < half; j++)
        for (uint32_t pos = 0; pos < max_seq; pos++) {
            t[((size_t)pos * half + j) * 2] = (float)std::cos(pos * freqs[j]), t[((size_t)pos * half + j) * 2 + 1] = (float)std::sin(pos * freqs[j]);
        }
    return t;
}
inline std::vector<double> rope_frequencies(double base, uint32_t dims) {
    std::vector<double> f(dims / 2);
    for (uint32_t j = 0; j < dims / 2; j++) f[j] = std::pow(base, -2.0 * j / dims);
    return f;
}

// ---- the frame of a model class -------------------------------------------------------------------------------------------------

// A piece of a sequence's state on the device.
struct StatePiece {
    void* d;
    size_t bytes;
};

// The norm in front of a product: a scalar and, when given, a gain per coordinate.
struct Gain {
    float g = 1.0f;
    const float* w = nullptr;
};

struct FolderModel : wick_rocm_model {
    bool f32 = false;
    uint32_t dp = 0, vp = 0;    // width / vocabulary padded
    float eps = 0.0f, embed_scale = 1.0f;
    uint16_t* embed = nullptr;
    DenseWeight head;
    Gain final_norm;
    std::vector<void*> buffers;
    size_t bytes = 0;
    bool use_graph = true;
    wick_rocm_graph* graphs[kStepModes] = {};
    std::map<std::vector<double>, float*> ropes;  // tables by their frequencies
    // a step's vectors
    float *x0 = nullptr, *xs[2] = {}, *logits = nullptr;
    uint32_t *d_token = nullptr, *d_pos = nullptr, *d_pick = nullptr, *d_history = nullptr;
    unsigned long long* d_partial = nullptr;
    // a prompt pass's rows, allocated by the first one
    uint32_t cap = 0;
    uint32_t *p_tokens = nullptr, *p_rows = nullptr;
    float *p_x0 = nullptr, *p_x[2] = {}, *p_logits = nullptr, *p_trace = nullptr;
    void* p_h = nullptr;

    // One step's launches: token and position are read on the device, x0 holds the token's embedding row already.
    virtual int enqueue_step(wick_rocm_ctx* ctx, StepMode mode) = 0;
    // Allocates what a prompt pass needs and sets `cap`; called when cap is 0.
    virtual int alloc_rows(wick_rocm_ctx* ctx) = 0;
    virtual int prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want,
                            float* logits_out, float* layers_out) = 0;
    virtual std::vector<StatePiece> state_pieces(uint32_t seq_len) const = 0;

    size_t act_bytes() const { return f32 ? 4 : 2; }

    int invalid(wick_rocm_ctx* ctx, int code, const std::string& what) {
        std::lock_guard<std::recursive_mutex> lk(ctx->mu);
        return fail(ctx, code, (std::string(info.architecture) + ": " + what).c_str());
    }
    int alloc(wick_rocm_ctx* ctx, size_t nbytes, void** out) {
        MODEL_TRY(wick_rocm_buffer_alloc(ctx, nbytes, out));
        buffers.push_back(*out);
        bytes += nbytes;
        return WICK_ROCM_OK;
    }
    template <typename T>
    int alloc_t(wick_rocm_ctx* ctx, size_t count, T** out) { return alloc(ctx, (count ? count : 1) * sizeof(T), reinterpret_cast<void**>(out)); }
    int alloc_act(wick_rocm_ctx* ctx, size_t count, void** out) { return alloc(ctx, (count ? count : 1) * act_bytes(), out); }
    int upload(wick_rocm_ctx* ctx, const Packer& p, DenseWeight* out) {
        MODEL_TRY(alloc_t(ctx, p.v.size(), &out->d));
        out->mp = p.mp, out->kp = p.kp, out->stride = p.stride;
        return wick_rocm_upload(ctx, out->d, p.v.data(), p.v.size() * 2);
    }
    template <typename T>
    int upload(wick_rocm_ctx* ctx, const std::vector<T>& v, T** out) {
        MODEL_TRY(alloc_t(ctx, v.size(), out));
        return v.empty() ? WICK_ROCM_OK : wick_rocm_upload(ctx, *out, v.data(), v.size() * sizeof(T));
    }
    int upload_rope(wick_rocm_ctx* ctx, const std::vector<double>& freqs, float** out) {
        float*& t = ropes[freqs];
        if (!t) MODEL_TRY(upload(ctx, rope_table(freqs, info.max_seq_len), &t));
        *out = t;
        return WICK_ROCM_OK;
    }
    // Sizes, the embedding and the head (head null: the embedding table itself).
    int load_ends(wick_rocm_ctx* ctx, const wick_safetensors* f, const char* architecture, uint32_t vocab, uint32_t width, uint32_t context_size, const char* head_name) {
        dp = pad_to(width, kDensePad), vp = pad_to(vocab, kDensePad);
        strcpy(info.architecture, architecture);
        info.vocab_size = vocab, info.hidden_size = width, info.max_seq_len = context_size;
        info.dtype = f32 ? WICK_ROCM_MODEL_F32 : WICK_ROCM_MODEL_NATIVE;
        const uint16_t* table = tensor(f, "embed", {vocab, width});
        Packer h(1, vocab, width);
        h.rows(0, 0, head_name ? tensor(f, head_name, {vocab, width}) : table, vocab, width);
        MODEL_TRY(upload(ctx, h, &head));
        if (!head_name && head.kp == width) {  // one copy serves both ends
            embed = head.d;
            return WICK_ROCM_OK;
        }
        std::vector<uint16_t> e((size_t)vocab * width);
        memcpy(e.data(), table, e.size() * 2);
        return upload(ctx, e, &embed);
    }
    int alloc_step(wick_rocm_ctx* ctx) {
        MODEL_TRY(alloc_t(ctx, dp, &x0));
        for (float*& x : xs) MODEL_TRY(alloc_t(ctx, dp, &x));
        MODEL_TRY(alloc_t(ctx, vp, &logits));
        MODEL_TRY(alloc_t(ctx, 1, &d_token));
        MODEL_TRY(alloc_t(ctx, 1, &d_pos));
        MODEL_TRY(alloc_t(ctx, 1, &d_pick));
        MODEL_TRY(alloc_t(ctx, kArgmaxPartials, &d_partial));
        return alloc_t(ctx, info.max_seq_len, &d_history);
    }
    int alloc_pass(wick_rocm_ctx* ctx, uint32_t n) {
        MODEL_TRY(alloc_t(ctx, n, &p_tokens));
        MODEL_TRY(alloc_t(ctx, n, &p_rows));
        MODEL_TRY(alloc_t(ctx, (size_t)n * dp, &p_x0));
        for (float*& x : p_x) MODEL_TRY(alloc_t(ctx, (size_t)n * dp, &x));
        MODEL_TRY(alloc_t(ctx, (size_t)kHeadRows * vp, &p_logits));
        return alloc_act(ctx, (size_t)n * dp, &p_h);
    }

    void release(wick_rocm_ctx* ctx) override {
        wick_rocm_sync(ctx);
        for (wick_rocm_graph*& g : graphs)
            if (g) wick_rocm_graph_destroy(ctx, g), g = nullptr;
        for (void* b : buffers) wick_rocm_buffer_free(ctx, b);
        buffers.clear();
    }
    size_t memory_bytes() const override { return bytes; }
    void set_graph_replay(bool on) override { use_graph = on; }
    int reset(wick_rocm_ctx*) override { return WICK_ROCM_OK; }  // nothing carries over to a sequence that starts at position 0

    int run_step(wick_rocm_ctx* ctx, StepMode mode) {
        return run_step_graph(ctx, graphs[mode], use_graph, [&] { return enqueue_step(ctx, mode); });
    }
    int set_step(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos) {
        MODEL_LAUNCH(launch_set_step(d_token, token, d_pos, pos, ctx->launch(), reinterpret_cast<const uint8_t*>(embed), kTypeBF16, info.vocab_size,
                                     info.hidden_size, x0, embed_scale));
        return WICK_ROCM_OK;
    }
    // The last launches of a step: the head over the finished residual (in.row) and the pick.
    int finish_step(wick_rocm_ctx* ctx, StepMode mode, const GemvIn& in) {
        if (mode == kStepNoHead) return WICK_ROCM_OK;
        const Launch L = ctx->launch();
        MODEL_LAUNCH(launch_gemv_dense(head, info.vocab_size, in, logits, nullptr, kActNone, 0, L));
        if (mode == kStepGreedy)
            MODEL_LAUNCH(launch_argmax(logits, info.vocab_size, d_partial, d_pick, d_token, d_pos, d_history, info.max_seq_len, L,
                                       reinterpret_cast<const uint8_t*>(embed), kTypeBF16, info.vocab_size, info.hidden_size, x0, embed_scale));
        return WICK_ROCM_OK;
    }
    int generate(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out) override {
        MODEL_TRY(set_step(ctx, token, pos));
        for (uint32_t i = 0; i < n; i++) MODEL_TRY(run_step(ctx, kStepGreedy));
        return wick_rocm_download(ctx, out, d_history + pos, (size_t)n * sizeof(uint32_t));
    }
    int forward(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos, const uint32_t* want, uint32_t n_want, float* logits_out,
                float* layers_out) override {
        const size_t vocab = info.vocab_size;
        uint32_t w = 0;
        if (n <= kStepsMax && !layers_out) {
            for (uint32_t i = 0; i < n; i++) {
                const bool wanted = w < n_want && want[w] == i;
                MODEL_TRY(set_step(ctx, tokens[i], pos + i));
                MODEL_TRY(run_step(ctx, wanted ? kStepLogits : kStepNoHead));
                if (wanted) MODEL_TRY(wick_rocm_download(ctx, logits_out + w++ * vocab, logits, vocab * sizeof(float)));
            }
            return wick_rocm_sync(ctx);
        }
        if (!cap) MODEL_TRY(alloc_rows(ctx));
        if (layers_out && n > cap) return invalid(ctx, WICK_ROCM_ERR_INVALID_ARG, "per-layer copies: more tokens than one prompt pass takes");
        for (uint32_t at = 0; at < n; at += cap) {
            const uint32_t count = std::min(cap, n - at);
            std::vector<uint32_t> here;
            const uint32_t w0 = w;
            while (w < n_want && want[w] < at + count) here.push_back(want[w++] - at);
            MODEL_TRY(prompt_pass(ctx, tokens + at, count, pos + at, here.data(), (uint32_t)here.size(), logits_out + w0 * vocab, layers_out));
        }
        return wick_rocm_sync(ctx);
    }
    // The residual update and norm of n rows; `pend` is the sublayers' output that is still to be added to x.
    RowsArgs rows_of(const RowStage& pend, const float* x, const Gain& pre, bool keep, uint32_t n, uint32_t pos0) const {
        RowsArgs a;
        a.s = pend;
        a.s.x = x, a.s.x_stride = dp, a.s.y_stride = dp, a.s.g_pre = pre.g, a.s.w_pre = pre.w, a.s.eps = eps, a.s.dim = info.hidden_size;
        if (keep && pend.pending()) a.s.x_out = x == p_x[0] ? p_x[1] : p_x[0];
        a.n = n, a.pos0 = pos0, a.out = p_h, a.ldo = dp, a.kp = dp, a.f32 = f32;
        return a;
    }
    // The residual stream as it stands, [n][hidden], to the host.
    int copy_residual(wick_rocm_ctx* ctx, const RowStage& pend, const float* x, uint32_t n, float* out) {
        const uint32_t D = info.hidden_size;
        const float* from = x;
        if (pend.pending()) {
            if (!p_trace) MODEL_TRY(alloc_t(ctx, (size_t)cap * dp, &p_trace));
            RowsArgs a = rows_of(pend, x, Gain(), false, n, 0);
            a.s.x_out = p_trace;
            MODEL_LAUNCH(launch_rows(a, kRowOnly, ctx->launch()));
            from = p_trace;
        }
        std::vector<float> host((size_t)n * dp);
        MODEL_TRY(wick_rocm_download(ctx, host.data(), from, host.size() * sizeof(float)));
        for (uint32_t t = 0; t < n; t++) memcpy(out + (size_t)t * D, &host[(size_t)t * dp], (size_t)D * sizeof(float));
        return WICK_ROCM_OK;
    }
    // Logits of the wanted rows of a pass.
    int wanted_logits(wick_rocm_ctx* ctx, const RowStage& pend, const float* x, const uint32_t* want, uint32_t n_want, float* logits_out) {
        if (n_want == 0) return WICK_ROCM_OK;
        const Launch L = ctx->launch();
        const size_t vocab = info.vocab_size;
        MODEL_TRY(wick_rocm_upload(ctx, p_rows, want, (size_t)n_want * sizeof(uint32_t)));
        if (n_want <= kHeadGemvRows) {
            RowsArgs a = rows_of(pend, x, Gain(), true, n_want, 0);
            a.rows = p_rows;
            if (a.s.x_out) {  // the wanted rows of the finished residual
                MODEL_LAUNCH(launch_rows(a, kRowOnly, L));
                x = a.s.x_out;
            }
            for (uint32_t i = 0; i < n_want; i++) {
                GemvIn in;
                in.row.x = x + (size_t)want[i] * dp, in.row.x_stride = dp, in.row.g_pre = final_norm.g, in.row.w_pre = final_norm.w;
                in.row.eps = eps, in.row.dim = info.hidden_size;
                MODEL_LAUNCH(launch_gemv_dense(head, info.vocab_size, in, p_logits + (size_t)i * vp, nullptr, kActNone, 0, L));
            }
            for (uint32_t i = 0; i < n_want; i++) MODEL_TRY(wick_rocm_download(ctx, logits_out + i * vocab, p_logits + (size_t)i * vp, vocab * sizeof(float)));
            return WICK_ROCM_OK;
        }
        std::vector<float> host;
        for (uint32_t first = 0; first < n_want; first += kHeadRows) {
            const uint32_t count = std::min(kHeadRows, n_want - first);
            RowsArgs a = rows_of(pend, x, final_norm, false, count, 0);
            a.rows = p_rows + first;
            MODEL_LAUNCH(launch_rows(a, kRowNorm, L));
            MODEL_LAUNCH(launch_gemm_store(head, GemmIn{p_h, dp, count, f32}, p_logits, vp, nullptr, L));
            host.resize((size_t)count * vp);
            MODEL_TRY(wick_rocm_download(ctx, host.data(), p_logits, host.size() * sizeof(float)));
            for (uint32_t i = 0; i < count; i++) memcpy(logits_out + (first + i) * vocab, &host[(size_t)i * vp], vocab * sizeof(float));
        }
        return WICK_ROCM_OK;
    }

    size_t state_bytes(uint32_t seq_len) const override {
        size_t total = 0;
        for (const StatePiece& p : state_pieces(seq_len)) total += p.bytes;
        return total;
    }
    int snapshot(wick_rocm_ctx* ctx, uint32_t seq_len, void* out) override {
        char* at = static_cast<char*>(out);
        for (const StatePiece& p : state_pieces(seq_len)) {
            MODEL_TRY(wick_rocm_download(ctx, at, p.d, p.bytes));
            at += p.bytes;
        }
        return WICK_ROCM_OK;
    }
    int restore(wick_rocm_ctx* ctx, uint32_t seq_len, const void* in) override {
        const char* at = static_cast<const char*>(in);
        for (const StatePiece& p : state_pieces(seq_len)) {
            MODEL_TRY(wick_rocm_upload(ctx, p.d, at, p.bytes));
            at += p.bytes;
        }
        return WICK_ROCM_OK;
    }
};

// A loader for the registry: load() says what does not fit by throwing ConfigError.
template <typename M>
int load_folder_model(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out) {
    std::unique_ptr<M> m(new M);
    m->f32 = dtype == WICK_ROCM_MODEL_F32;
    int rc;
    try {
        rc = m->load(ctx, folder, context_size);
    } catch (const ConfigError& e) {
        rc = m->invalid(ctx, WICK_ROCM_ERR_BAD_SHAPE, e.what);
    }
    if (rc) {
        m->release(ctx);
        return rc;
    }
    *out = m.release();
    return WICK_ROCM_OK;
}

}  // namespace folder_model
