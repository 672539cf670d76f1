// The Lokinex model: config.json and tensors of a model folder -> packed weights, caches and states -> steps and prompt passes over
// the kernels of wick_rocm_dense.h.  Host code only.
//
// A decoder whose layers mix with a real-gated linear recurrence or with attention over a cached latent, behind a short convolution of
// the layer's input; norms with one gain before and after every sublayer; dense (squared ReLU) or table-routed feed-forwards; and a
// stretch of layers that a token goes through several times, each pass with caches of its own and the embedding mixed in at its start.
//
// State of a sequence, per layer run: the ring of the last inputs of the layer's convolution and, by type, the latent cache or the
// ring of the block's own convolution with the recurrent state.  Rings are addressed by position and a recurrent state is only read
// past position 0, so a sequence that starts at position 0 needs nothing cleared.
#include <cmath>
#include <cstring>
#include <map>
#include <memory>
#include <vector>

#include "model.h"
#include "model_folder.h"
#include "wick_rocm_dense.h"

namespace {

constexpr uint32_t kChunkBf16 = 2048, kChunkExact = 512;  // tokens per prompt pass: bfloat16 / f32 or a head shape without matrix-core attention
constexpr uint32_t kStepsMax = 2;       // portions this short run as single steps
constexpr uint32_t kAbsorbMax = 16;     // ... this short attend with absorbed queries, without expanding the cache
constexpr uint32_t kHeadRows = 64;      // wanted rows per product with the head
constexpr uint32_t kHeadGemvRows = 4;   // up to this many run as matrix-vector products

struct MixerConfig {
    bool recurrent = false;
    uint32_t width = 0, blocks = 0, conv = 0;                        // rglru
    uint32_t heads = 0, dim = 0, rot = 0, vdim = 0, rank = 0;        // latent_attention
    double rope_base = 0.0, scale = 0.0;
};
struct MlpConfig {
    enum Kind { kNone, kDense, kMoe } kind = kNone;
    uint32_t ff = 0, experts = 0, top = 0, shared_ff = 0;
};
struct Config {
    uint32_t vocab = 0, width = 0, taps = 0, loop_start = 0, loop_stop = 0, loop_times = 0;
    double eps = 0.0;
    std::vector<std::pair<MixerConfig, MlpConfig>> layers;
};

struct Layer {
    MixerConfig mix;
    MlpConfig mlp;
    float norm1 = 0, norm1b = 0, norm2 = 0, norm2b = 0;
    float* canon = nullptr;   // [taps][dp]
    DenseWeight in, out;
    // rglru: channels in blocks padded to `block`
    uint32_t block = 0, channels = 0;
    DenseWeight gates;
    float *in_bias = nullptr, *conv = nullptr, *conv_bias = nullptr, *r_bias = nullptr, *i_bias = nullptr, *rate = nullptr;
    // latent attention
    LatentShape shape{};
    LatentWeights lat{};
    DenseWeight kx, vx;
    uint32_t dqp = 0, dvp = 0;  // 0: no matrix-core prefill for this head shape
    // feed-forward
    DenseWeight up, down;
    RoutedMlp moe;
    uint32_t job = 0;           // of its table among the routing jobs
    uint32_t *entry_token = nullptr, *slot_of = nullptr, *n_tiles = nullptr;
    GroupTile* tiles = nullptr;
};

struct Run {
    uint32_t layer = 0;
    int pass = -1;              // >= 0: the loop's entry comes first
    float *canon_ring = nullptr, *conv_ring = nullptr, *state = nullptr;
    void* cache = nullptr;
};

enum StepMode { kStepLogits = 0, kStepGreedy = 1, kStepNoHead = 2, kStepModes = 3 };

struct Lokinex final : wick_rocm_model {
    Config cfg;
    bool f32 = false;
    uint32_t dp = 0, vp = 0;    // width / vocabulary padded
    uint16_t* embed = nullptr;
    DenseWeight head, loop_in;
    float* loop_step = nullptr; // [times][dp]
    float final_norm = 0;
    std::vector<Layer> layers;
    std::vector<Run> runs;
    std::vector<void*> buffers;
    size_t bytes = 0;
    bool use_graph = true;
    wick_rocm_graph* graphs[kStepModes] = {};
    // a step's vectors
    float *x0 = nullptr, *xs[2] = {}, *y = nullptr, *proj = nullptr, *mixed = nullptr, *act = nullptr, *qa = nullptr, *scratch = nullptr, *logits = nullptr;
    uint32_t *d_token = nullptr, *d_pos = nullptr, *d_pick = nullptr, *d_history = nullptr;
    unsigned long long* d_partial = nullptr;
    // a prompt pass's rows, allocated by the first one
    uint32_t cap = 0;
    uint32_t *p_tokens = nullptr, *p_rows = nullptr;
    float *p_x0 = nullptr, *p_x[2] = {}, *p_y = nullptr, *p_ye = nullptr, *p_proj = nullptr, *p_gate = nullptr, *p_u = nullptr, *p_a = nullptr, *p_b = nullptr,
          *p_qa = nullptr, *p_scratch = nullptr, *p_logits = nullptr, *p_trace = nullptr;
    void *p_loop = nullptr, *p_h = nullptr, *p_mixed = nullptr, *p_act = nullptr, *p_acte = nullptr, *p_ua = nullptr;
    uint16_t *p_q = nullptr, *p_kx = nullptr, *p_vt = nullptr;
    RouteJob* p_jobs = nullptr;
    uint32_t n_jobs = 0, absorb_cap = 0;

    size_t act_bytes() const { return f32 ? 4 : 2; }
    uint32_t loop_terms() const { return f32 ? 2 : 3; }  // columns of the loop's input in units of dp: x (hi) | x0 (| x lo)
    uint32_t kv_pad() const { return pad_to(info.max_seq_len, 64); }

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
    int forward(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos, const uint32_t* want, uint32_t n_want, float* logits_out,
                float* layers_out) override;
    int generate(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out) override;
    size_t state_bytes(uint32_t seq_len) const override;
    int snapshot(wick_rocm_ctx* ctx, uint32_t seq_len, void* out) override;
    int restore(wick_rocm_ctx* ctx, uint32_t seq_len, const void* in) override;

    int load(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t context_size);
    int alloc(wick_rocm_ctx* ctx, size_t nbytes, void** out);
    template <typename T>
    int alloc_t(wick_rocm_ctx* ctx, size_t count, T** out) { return alloc(ctx, (count ? count : 1) * sizeof(T), reinterpret_cast<void**>(out)); }
    int alloc_rows(wick_rocm_ctx* ctx);
    int load_layer(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t i, std::map<std::pair<uint32_t, double>, float*>& ropes);
    int set_step(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos);
    int enqueue_step(wick_rocm_ctx* ctx, StepMode mode);
    int run_step(wick_rocm_ctx* ctx, StepMode mode) {
        return run_step_graph(ctx, graphs[mode], use_graph, [&] { return enqueue_step(ctx, mode); });
    }
    int prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                    float* layers_out);
    int prompt_mixer(wick_rocm_ctx* ctx, const Layer& l, const Run& r, uint32_t n, uint32_t pos0);
    int prompt_mlp(wick_rocm_ctx* ctx, const Layer& l, uint32_t n);
    template <typename F>
    int for_each_state_piece(uint32_t seq_len, F&& piece) const;
};

int ctx_fail(wick_rocm_ctx* ctx, int code, const std::string& what) {
    std::lock_guard<std::recursive_mutex> lk(ctx->mu);
    return fail(ctx, code, ("lokinex: " + what).c_str());
}

#define LK_LAUNCH(call)                                                       \
    do {                                                                      \
        const hipError_t e_ = (call);                                         \
        if (e_ != hipSuccess) return fail_hip(ctx, e_, "lokinex: " #call);    \
    } while (0)
#define LK_TRY(call)                      \
    do {                                  \
        if (int rc_ = (call)) return rc_; \
    } while (0)

// ---- config.json ------------------------------------------------------------------------------------------------------------

struct ConfigError {
    std::string what;
};

const Json& need(const Json& j, const char* key, const std::string& where) {
    const Json* v = j.find(key);
    if (!v) throw ConfigError{"config: " + where + " has no \"" + key + "\""};
    return *v;
}
double number(const Json& j, const char* key, const std::string& where) {
    const Json& v = need(j, key, where);
    if (v.kind != Json::kNumber || !std::isfinite(v.number)) throw ConfigError{"config: " + where + "." + key + " is not a number"};
    return v.number;
}
uint32_t size(const Json& j, const char* key, const std::string& where, uint32_t least = 1) {
    const double v = number(j, key, where);
    if (v < least || v > 1e9 || v != std::floor(v)) throw ConfigError{"config: " + where + "." + key + " is out of range"};
    return (uint32_t)v;
}
const std::string& text(const Json& j, const char* key, const std::string& where) {
    const Json& v = need(j, key, where);
    if (v.kind != Json::kString) throw ConfigError{"config: " + where + "." + key + " is not a string"};
    return v.string;
}

MixerConfig mixer_config(const Json& layer, const std::string& where) {
    MixerConfig m;
    const std::string& type = text(layer, "type", where);
    const Json& j = need(layer, "mixer", where);
    const std::string w = where + ".mixer";
    if (type == "rglru") {
        m.recurrent = true;
        m.width = size(j, "width", w), m.blocks = size(j, "blocks", w), m.conv = size(j, "conv", w);
        if (m.width % m.blocks) throw ConfigError{"config: " + w + ": blocks must divide width"};
    } else if (type == "latent_attention") {
        m.heads = size(j, "heads", w), m.dim = size(j, "dim", w), m.rot = size(j, "rot_dim", w), m.vdim = size(j, "vdim", w), m.rank = size(j, "kv_rank", w);
        m.scale = number(j, "scale", w);
        const Json& r = need(j, "rot", w);
        m.rope_base = number(r, "base", w + ".rot");
        if (size(r, "dims", w + ".rot") != m.rot || m.rot % 2u) throw ConfigError{"config: " + w + ": rot.dims must be rot_dim, an even number"};
        if (!(m.rope_base > 0.0)) throw ConfigError{"config: " + w + ": rot.base must be positive"};
    } else {
        throw ConfigError{"config: " + where + ": unknown type " + type};
    }
    return m;
}

MlpConfig mlp_config(const Json& layer, const std::string& where) {
    MlpConfig c;
    const Json* j = layer.find("mlp");
    if (!j || j->is_null()) return c;
    const std::string w = where + ".mlp", &kind = text(*j, "kind", w);
    if (kind == "dense") {
        c.kind = MlpConfig::kDense, c.ff = size(*j, "ff", w);
    } else if (kind == "moe") {
        c.kind = MlpConfig::kMoe;
        c.ff = size(need(*j, "expert", w), "ff", w + ".expert");
        const Json& r = need(*j, "router", w);
        c.experts = size(r, "experts", w + ".router"), c.top = size(r, "top", w + ".router");
        if (c.top > c.experts) throw ConfigError{"config: " + w + ": more experts per token than experts"};
        const Json* s = j->find("shared");
        if (s && !s->is_null()) c.shared_ff = size(*s, "ff", w + ".shared");
    } else {
        throw ConfigError{"config: " + w + ": unknown kind " + kind};
    }
    return c;
}

Config read_config(const Json& j) {
    Config c;
    c.vocab = size(j, "vocab", "config"), c.width = size(j, "width", "config");
    c.taps = size(need(j, "canon", "config"), "taps", "canon");
    c.eps = number(need(j, "norm", "config"), "eps", "norm");
    const Json& layers = need(j, "layers", "config");
    if (layers.kind != Json::kArray || layers.items.empty()) throw ConfigError{"config: layers is not a list"};
    for (size_t i = 0; i < layers.items.size(); i++) {
        const std::string where = "layers[" + std::to_string(i) + "]";
        c.layers.emplace_back(mixer_config(layers.items[i], where), mlp_config(layers.items[i], where));
    }
    const Json* loop = j.find("loop");
    if (loop && !loop->is_null()) {
        c.loop_start = size(*loop, "start", "loop", 0), c.loop_stop = size(*loop, "stop", "loop"), c.loop_times = size(*loop, "times", "loop");
        if (c.loop_start >= c.loop_stop || c.loop_stop > c.layers.size()) throw ConfigError{"config: loop does not lie inside the layers"};
    }
    return c;
}

// ---- weights ----------------------------------------------------------------------------------------------------------------

float bf16(uint16_t b) {
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

// A bfloat16 tensor of the given shape.
const uint16_t* tensor(const wick_safetensors* f, const std::string& name, const std::vector<uint64_t>& shape) {
    const wick_safetensors::Tensor* t = f->find(name);
    if (!t) throw ConfigError{"no tensor " + name};
    if (t->dtype != WICK_SAFETENSORS_BF16 || t->shape != shape) throw ConfigError{"tensor " + name + " has another type or shape than the config says"};
    return reinterpret_cast<const uint16_t*>(t->data);
}
float scalar(const wick_safetensors* f, const std::string& name) { return bf16(*tensor(f, name, {})); }

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

int upload(wick_rocm_ctx* ctx, Lokinex* m, const Packer& p, DenseWeight* out) {
    LK_TRY(m->alloc_t(ctx, p.v.size(), &out->d));
    out->mp = p.mp, out->kp = p.kp, out->stride = p.stride;
    return wick_rocm_upload(ctx, out->d, p.v.data(), p.v.size() * 2);
}
int upload(wick_rocm_ctx* ctx, Lokinex* m, const std::vector<float>& v, float** out) {
    LK_TRY(m->alloc_t(ctx, v.size(), out));
    return wick_rocm_upload(ctx, *out, v.data(), v.size() * 4);
}
int upload(wick_rocm_ctx* ctx, Lokinex* m, const std::vector<uint16_t>& v, uint16_t** out) {
    LK_TRY(m->alloc_t(ctx, v.size(), out));
    return wick_rocm_upload(ctx, *out, v.data(), v.size() * 2);
}

int Lokinex::alloc(wick_rocm_ctx* ctx, size_t nbytes, void** out) {
    LK_TRY(wick_rocm_buffer_alloc(ctx, nbytes, out));
    buffers.push_back(*out);
    bytes += nbytes;
    return WICK_ROCM_OK;
}

int Lokinex::load_layer(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t i, std::map<std::pair<uint32_t, double>, float*>& ropes) {
    const std::string p = "l" + std::to_string(i) + ".", mp = p + "mix.", fp = p + "mlp.";
    Layer& l = layers[i];
    const uint32_t D = cfg.width;
    const MixerConfig& m = l.mix = cfg.layers[i].first;
    const MlpConfig& c = l.mlp = cfg.layers[i].second;
    l.norm1 = scalar(f, p + "norm1"), l.norm1b = scalar(f, p + "norm1b");
    {
        const uint16_t* w = tensor(f, p + "canon1", {D, cfg.taps});
        std::vector<float> v((size_t)cfg.taps * dp, 0.0f);
        for (uint32_t e = 0; e < D; e++)
            for (uint32_t k = 0; k < cfg.taps; k++) v[(size_t)k * dp + e] = bf16(w[(size_t)e * cfg.taps + k]);
        LK_TRY(upload(ctx, this, v, &l.canon));
    }
    if (m.recurrent) {
        // channels go by block, every block padded to a multiple of 64: channel b * bs + j sits at b * block + j
        const uint32_t W = m.width, bs = W / m.blocks, bp = pad_to(bs, kDensePad), C = m.blocks * bp;
        l.block = bp, l.channels = C;
        auto at = [&](uint32_t ch) { return ch / bs * bp + ch % bs; };
        auto spread = [&](const uint16_t* src) {
            std::vector<float> v(C, 0.0f);
            for (uint32_t ch = 0; ch < W; ch++) v[at(ch)] = bf16(src[ch]);
            return v;
        };
        {
            Packer w(1, 2 * C, D);
            const uint16_t *wy = tensor(f, mp + "y", {W, D}), *wx = tensor(f, mp + "x", {W, D});
            for (uint32_t ch = 0; ch < W; ch++) w.row(0, at(ch), wy + (size_t)ch * D, D), w.row(0, C + at(ch), wx + (size_t)ch * D, D);
            LK_TRY(upload(ctx, this, w, &l.in));
            std::vector<float> b = spread(tensor(f, mp + "y.b", {W})), bx = spread(tensor(f, mp + "x.b", {W}));
            b.insert(b.end(), bx.begin(), bx.end());
            LK_TRY(upload(ctx, this, b, &l.in_bias));
        }
        {
            const uint16_t* w = tensor(f, mp + "conv", {W, m.conv});
            std::vector<float> v((size_t)m.conv * C, 0.0f);
            for (uint32_t ch = 0; ch < W; ch++)
                for (uint32_t k = 0; k < m.conv; k++) v[(size_t)k * C + at(ch)] = bf16(w[(size_t)ch * m.conv + k]);
            LK_TRY(upload(ctx, this, v, &l.conv));
            LK_TRY(upload(ctx, this, spread(tensor(f, mp + "conv.b", {W})), &l.conv_bias));
        }
        {
            // bfloat16 products take u as two terms: the block's columns once per term
            const uint32_t terms = f32 ? 1 : 2;
            Packer w(m.blocks, 2 * bp, terms * bp);
            const uint16_t *ra = tensor(f, mp + "ra", {m.blocks, bs, bs}), *ri = tensor(f, mp + "ri", {m.blocks, bs, bs});
            for (uint32_t b = 0; b < m.blocks; b++)
                for (uint32_t t = 0; t < terms; t++) w.pair(b, ra + (size_t)b * bs * bs, ri + (size_t)b * bs * bs, bs, bs, t * bp);
            LK_TRY(upload(ctx, this, w, &l.gates));
            LK_TRY(upload(ctx, this, spread(tensor(f, mp + "ra.b", {m.blocks, bs})), &l.r_bias));
            LK_TRY(upload(ctx, this, spread(tensor(f, mp + "ri.b", {m.blocks, bs})), &l.i_bias));
            std::vector<float> rate(C, 0.0f);
            const uint16_t* lam = tensor(f, mp + "lam", {W});
            for (uint32_t ch = 0; ch < W; ch++) {
                const double z = bf16(lam[ch]);
                rate[at(ch)] = (float)(-8.0 * (std::fmax(z, 0.0) + std::log1p(std::exp(-std::fabs(z)))));  // -8 softplus(lam)
            }
            LK_TRY(upload(ctx, this, rate, &l.rate));
        }
        Packer o(1, D, C);
        const uint16_t* wo = tensor(f, mp + "o", {D, W});
        for (uint32_t r = 0; r < D; r++)
            for (uint32_t b = 0; b < m.blocks; b++) o.row(0, r, wo + (size_t)r * W + b * bs, bs, b * bp);
        LK_TRY(upload(ctx, this, o, &l.out));
    } else {
        LatentShape& s = l.shape;
        s.heads = m.heads, s.dim = m.dim, s.rot = m.rot, s.vdim = m.vdim, s.rank = m.rank;
        s.rank_p = pad_to(m.rank, 32), s.rot_p = pad_to(m.rot, 32);
        if (s.row() % 64u) s.rot_p += 32;
        s.scale = (float)m.scale, s.eps = (float)cfg.eps, s.max_seq = info.max_seq_len, s.f32 = f32;
        const uint32_t H = m.heads, qrows = H * (m.dim + m.rot);
        Packer w(1, qrows + m.rank + m.rot, D);
        w.rows(0, 0, tensor(f, mp + "q", {qrows, D}), qrows, D);
        w.rows(0, qrows, tensor(f, mp + "dkv", {m.rank + m.rot, D}), m.rank + m.rot, D);
        LK_TRY(upload(ctx, this, w, &l.in));
        const uint16_t *uk = tensor(f, mp + "uk", {H * m.dim, m.rank}), *uv = tensor(f, mp + "uv", {H * m.vdim, m.rank});
        auto padded = [&](const uint16_t* src, uint32_t rows) {
            std::vector<uint16_t> v((size_t)rows * s.rank_p, 0);
            for (uint32_t r = 0; r < rows; r++) memcpy(&v[(size_t)r * s.rank_p], src + (size_t)r * m.rank, (size_t)m.rank * 2);
            return v;
        };
        uint16_t *d_uk = nullptr, *d_uv = nullptr;
        LK_TRY(upload(ctx, this, padded(uk, H * m.dim), &d_uk));
        LK_TRY(upload(ctx, this, padded(uv, H * m.vdim), &d_uv));
        std::vector<float> norm(m.rank);
        const uint16_t* nw = tensor(f, mp + "dkv.norm", {m.rank});
        for (uint32_t e = 0; e < m.rank; e++) norm[e] = bf16(nw[e]);
        float* d_norm = nullptr;
        LK_TRY(upload(ctx, this, norm, &d_norm));
        float*& rope = ropes[{m.rot, m.rope_base}];
        if (!rope) {
            const uint32_t half = m.rot / 2;
            std::vector<float> t((size_t)info.max_seq_len * half * 2);
            for (uint32_t j = 0; j < half; j++) {
                const double freq = std::pow(m.rope_base, -2.0 * j / m.rot);
                for (uint32_t pos = 0; pos < info.max_seq_len; pos++) {
                    t[((size_t)pos * half + j) * 2] = (float)std::cos(pos * freq), t[((size_t)pos * half + j) * 2 + 1] = (float)std::sin(pos * freq);
                }
            }
            LK_TRY(upload(ctx, this, t, &rope));
        }
        l.lat = LatentWeights{d_uk, d_uv, d_norm, rope};
        if (!f32 && latent_prefill_shape(m.dim, m.rot, m.vdim, &l.dqp, &l.dvp)) {
            // keys and values of a cache row as plain products over it: the rotated part is copied by ones
            const uint16_t one = 0x3f80;
            Packer k(1, H * l.dqp, s.row()), v(1, H * l.dvp, s.row());
            for (uint32_t h = 0; h < H; h++) {
                k.rows(0, h * l.dqp, uk + (size_t)h * m.dim * m.rank, m.dim, m.rank);
                for (uint32_t j = 0; j < m.rot; j++) k.row(0, h * l.dqp + m.dim + j, &one, 1, s.rank_p + j);
                v.rows(0, h * l.dvp, uv + (size_t)h * m.vdim * m.rank, m.vdim, m.rank);
            }
            LK_TRY(upload(ctx, this, k, &l.kx));
            LK_TRY(upload(ctx, this, v, &l.vx));
        } else {
            l.dqp = l.dvp = 0;
        }
        Packer o(1, D, H * m.vdim);
        o.rows(0, 0, tensor(f, mp + "o", {D, H * m.vdim}), D, H * m.vdim);
        LK_TRY(upload(ctx, this, o, &l.out));
    }
    if (c.kind == MlpConfig::kNone) return WICK_ROCM_OK;
    l.norm2 = scalar(f, p + "norm2"), l.norm2b = scalar(f, p + "norm2b");
    if (c.kind == MlpConfig::kDense) {
        Packer up(1, c.ff, D), down(1, D, c.ff);
        up.rows(0, 0, tensor(f, fp + "up", {c.ff, D}), c.ff, D);
        down.rows(0, 0, tensor(f, fp + "down", {D, c.ff}), D, c.ff);
        LK_TRY(upload(ctx, this, up, &l.up));
        return upload(ctx, this, down, &l.down);
    }
    RoutedMlp& r = l.moe;
    r.top = c.top, r.experts = c.experts;
    {
        Packer gu(c.experts, 2 * pad_to(c.ff, kDensePad), D), down(c.experts, D, c.ff);
        for (uint32_t e = 0; e < c.experts; e++) {
            const std::string ep = fp + "e" + std::to_string(e) + ".";
            gu.pair(e, tensor(f, ep + "gate", {c.ff, D}), tensor(f, ep + "up", {c.ff, D}), c.ff, D);
            down.rows(e, 0, tensor(f, ep + "down", {D, c.ff}), D, c.ff);
        }
        LK_TRY(upload(ctx, this, gu, &r.gate_up));
        LK_TRY(upload(ctx, this, down, &r.down));
    }
    if (c.shared_ff) {
        Packer gu(1, 2 * pad_to(c.shared_ff, kDensePad), D), down(1, D, c.shared_ff), sg(1, 1, D);
        gu.pair(0, tensor(f, fp + "shared.gate", {c.shared_ff, D}), tensor(f, fp + "shared.up", {c.shared_ff, D}), c.shared_ff, D);
        down.rows(0, 0, tensor(f, fp + "shared.down", {D, c.shared_ff}), D, c.shared_ff);
        sg.row(0, 0, tensor(f, fp + "shared.sg", {1, D}), D);
        DenseWeight w;
        LK_TRY(upload(ctx, this, gu, &r.shared_gate_up));
        LK_TRY(upload(ctx, this, down, &r.shared_down));
        LK_TRY(upload(ctx, this, sg, &w));
        r.shared_sg = w.d;
    }
    const wick_safetensors::Tensor* t = f->find(fp + "table");
    if (!t || t->dtype != WICK_SAFETENSORS_I32 || t->shape != std::vector<uint64_t>{cfg.vocab, c.top})
        throw ConfigError{"tensor " + fp + "table is missing or has another type or shape than the config says"};
    std::vector<int32_t> table((size_t)cfg.vocab * c.top);
    memcpy(table.data(), t->data, table.size() * 4);
    for (int32_t e : table)
        if (e < 0 || (uint32_t)e >= c.experts) throw ConfigError{"tensor " + fp + "table names an expert that does not exist"};
    int32_t* d_table = nullptr;
    LK_TRY(alloc_t(ctx, table.size(), &d_table));
    LK_TRY(wick_rocm_upload(ctx, d_table, table.data(), table.size() * 4));
    r.table = d_table;
    l.job = n_jobs++;
    return WICK_ROCM_OK;
}

int Lokinex::load(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t context_size) {
    cfg = read_config(f->config);
    const uint32_t D = cfg.width;
    dp = pad_to(D, kDensePad), vp = pad_to(cfg.vocab, kDensePad);
    strcpy(info.architecture, "Lokinex");
    info.vocab_size = cfg.vocab, info.hidden_size = D, info.max_seq_len = context_size;
    info.dtype = f32 ? WICK_ROCM_MODEL_F32 : WICK_ROCM_MODEL_NATIVE;
    // what the kernels' on-chip buffers hold
    if (D > 7680u || D > rows_max_dim(cfg.taps) || cfg.taps > 16u) throw ConfigError{"width or canon.taps beyond what the kernels take"};
    for (const auto& l : cfg.layers) {
        const MixerConfig& m = l.first;
        const MlpConfig& c = l.second;
        const uint64_t routed = (uint64_t)c.top * pad_to(c.ff, kDensePad) + pad_to(c.shared_ff, kDensePad);
        const bool ok = m.recurrent ? (uint64_t)m.blocks * pad_to(m.width / m.blocks, kDensePad) <= 15360u && m.width / m.blocks <= 4096u && m.conv <= 8u
                                    : (uint64_t)m.heads * m.vdim <= 15360u && m.rank <= 2048u && m.rot <= 1024u && (uint64_t)m.heads * (m.dim + m.rot) <= 1u << 20;
        if (!ok || (c.kind == MlpConfig::kDense && c.ff > 15360u) || (c.kind == MlpConfig::kMoe && (routed > 15360u || c.experts > kRouteMaxExperts)))
            throw ConfigError{"a layer's sizes are beyond what the kernels take"};
    }

    std::vector<uint16_t> e((size_t)cfg.vocab * D);
    memcpy(e.data(), tensor(f, "embed", {cfg.vocab, D}), e.size() * 2);
    LK_TRY(upload(ctx, this, e, &embed));
    final_norm = scalar(f, "final.norm");
    {
        Packer h(1, cfg.vocab, D);
        h.rows(0, 0, tensor(f, "head", {cfg.vocab, D}), cfg.vocab, D);
        LK_TRY(upload(ctx, this, h, &head));
    }
    if (cfg.loop_times) {
        // [x | x0], and for bfloat16 products the low term of x behind them over the same columns of the weight
        Packer w(1, D, loop_terms() * dp);
        const uint16_t* src = tensor(f, "loop.in", {D, 2 * D});
        for (uint32_t r = 0; r < D; r++) {
            w.row(0, r, src + (size_t)r * 2 * D, D, 0), w.row(0, r, src + (size_t)r * 2 * D + D, D, dp);
            if (!f32) w.row(0, r, src + (size_t)r * 2 * D, D, 2 * dp);
        }
        LK_TRY(upload(ctx, this, w, &loop_in));
        const uint16_t* st = tensor(f, "loop.step", {cfg.loop_times, D});
        std::vector<float> v((size_t)cfg.loop_times * dp, 0.0f);
        for (uint32_t t = 0; t < cfg.loop_times; t++)
            for (uint32_t k = 0; k < D; k++) v[(size_t)t * dp + k] = bf16(st[(size_t)t * D + k]);
        LK_TRY(upload(ctx, this, v, &loop_step));
    }
    layers.resize(cfg.layers.size());
    std::map<std::pair<uint32_t, double>, float*> ropes;
    for (uint32_t i = 0; i < layers.size(); i++) LK_TRY(load_layer(ctx, f, i, ropes));

    // the order of the layer runs, every one with a state of its own
    auto push = [&](uint32_t layer, int pass) {
        runs.emplace_back();
        runs.back().layer = layer, runs.back().pass = pass;
    };
    if (!cfg.loop_times) cfg.loop_start = cfg.loop_stop = 0;
    for (uint32_t i = 0; i < cfg.loop_start; i++) push(i, -1);
    for (uint32_t t = 0; t < cfg.loop_times; t++)
        for (uint32_t i = cfg.loop_start; i < cfg.loop_stop; i++) push(i, i == cfg.loop_start ? (int)t : -1);
    for (uint32_t i = cfg.loop_stop; i < layers.size(); i++) push(i, -1);
    info.layer_runs = (uint32_t)runs.size();

    uint32_t proj_w = 4, mixed_w = 4, act_w = 4, qa_w = 4;
    size_t scratch_w = 4;
    for (Run& r : runs) {
        const Layer& l = layers[r.layer];
        LK_TRY(alloc_t(ctx, (size_t)cfg.taps * dp, &r.canon_ring));
        proj_w = std::max(proj_w, l.in.mp), mixed_w = std::max(mixed_w, l.out.kp);
        if (l.mix.recurrent) {
            LK_TRY(alloc_t(ctx, (size_t)l.mix.conv * l.channels, &r.conv_ring));
            LK_TRY(alloc_t(ctx, l.channels, &r.state));
        } else {
            LK_TRY(alloc(ctx, (size_t)info.max_seq_len * l.shape.row() * act_bytes(), &r.cache));
            qa_w = std::max(qa_w, l.shape.heads * l.shape.row());
            scratch_w = std::max(scratch_w, latent_attention_scratch_floats(l.shape, 1));
        }
        if (l.mlp.kind == MlpConfig::kDense) act_w = std::max(act_w, l.up.mp);
        if (l.mlp.kind == MlpConfig::kMoe) act_w = std::max(act_w, routed_act_floats(l.moe));
    }
    LK_TRY(alloc_t(ctx, dp, &x0));
    for (float*& x : xs) LK_TRY(alloc_t(ctx, dp, &x));
    LK_TRY(alloc_t(ctx, dp, &y));
    LK_TRY(alloc_t(ctx, proj_w, &proj));
    LK_TRY(alloc_t(ctx, mixed_w, &mixed));
    LK_TRY(alloc_t(ctx, act_w, &act));
    LK_TRY(alloc_t(ctx, qa_w, &qa));
    LK_TRY(alloc_t(ctx, scratch_w, &scratch));
    LK_TRY(alloc_t(ctx, vp, &logits));
    LK_TRY(alloc_t(ctx, 1, &d_token));
    LK_TRY(alloc_t(ctx, 1, &d_pos));
    LK_TRY(alloc_t(ctx, 1, &d_pick));
    LK_TRY(alloc_t(ctx, kArgmaxPartials, &d_partial));
    LK_TRY(alloc_t(ctx, info.max_seq_len, &d_history));
    return wick_rocm_sync(ctx);
}

// ---- one step ----------------------------------------------------------------------------------------------------------------

int Lokinex::set_step(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos) {
    LK_LAUNCH(launch_set_step(d_token, token, d_pos, pos, ctx->launch(), reinterpret_cast<const uint8_t*>(embed), kTypeBF16, cfg.vocab, cfg.width, x0));
    return WICK_ROCM_OK;
}

// Token and position are read on the device; x0 holds the token's embedding row already (set_step, or the previous greedy pick).
// The residual update behind a sublayer happens in the prologue of the launch that reads the residual next.
int Lokinex::enqueue_step(wick_rocm_ctx* ctx, StepMode mode) {
    const Launch L = ctx->launch();
    const uint32_t D = cfg.width;
    const float* x = x0;        // the residual, before ...
    const float* pending = nullptr;  // ... this sublayer output is added,
    float post = 0.0f;          // normed with this gain
    auto stage = [&](float g_pre) {
        RowStage s;
        s.x = x, s.x_stride = dp, s.y = pending, s.y_stride = dp, s.g_post = post, s.g_pre = g_pre, s.eps = (float)cfg.eps, s.dim = D;
        if (pending) s.x_out = x == xs[0] ? xs[1] : xs[0];
        return s;
    };
    auto staged = [&](const RowStage& s) {
        if (s.x_out) x = s.x_out;
        pending = nullptr;
    };
    for (const Run& r : runs) {
        const Layer& l = layers[r.layer];
        if (r.pass >= 0) {
            GemvIn in;
            in.row = stage(0.0f), in.row.x_out = nullptr;
            in.x0 = x0, in.x0_at = dp, in.k = 2 * dp;
            float* out = x == xs[0] ? xs[1] : xs[0];
            LK_LAUNCH(launch_gemv_dense(loop_in, D, in, out, loop_step + (size_t)r.pass * dp, kActNone, 0, L));
            x = out, pending = nullptr;
        }
        {
            GemvIn in;
            in.row = stage(l.norm1), in.d_pos = d_pos;
            in.row.conv = l.canon, in.row.ring = r.canon_ring, in.row.taps = cfg.taps;
            LK_LAUNCH(launch_gemv_dense(l.in, l.in.mp, in, proj, l.mix.recurrent ? l.in_bias : nullptr, l.mix.recurrent ? kActGeluSplit : kActNone, l.channels, L));
            staged(in.row);
        }
        if (l.mix.recurrent) {
            RecurrentStep s{};
            s.proj = proj, s.channels = l.channels, s.block = l.block, s.blocks = l.mix.blocks, s.taps = l.mix.conv;
            s.conv_w = l.conv, s.conv_bias = l.conv_bias, s.ring = r.conv_ring, s.state = r.state, s.gates = l.gates;
            s.r_bias = l.r_bias, s.i_bias = l.i_bias, s.rate = l.rate, s.out = mixed, s.d_pos = d_pos;
            LK_LAUNCH(launch_recurrent_step(s, L));
        } else {
            LK_LAUNCH(launch_latent_absorb(l.shape, l.lat, proj, l.in.mp, r.cache, qa, 1, 0, d_pos, L));
            LK_LAUNCH(launch_latent_attention(l.shape, l.lat, qa, r.cache, scratch, 1, 0, d_pos, mixed, l.out.kp, l.out.kp, true, L));
        }
        GemvIn mix;
        mix.vec = mixed;
        LK_LAUNCH(launch_gemv_dense(l.out, D, mix, y, nullptr, kActNone, 0, L));
        pending = y, post = l.norm1b;
        if (l.mlp.kind == MlpConfig::kNone) continue;
        GemvIn in;
        in.row = stage(l.norm2);
        if (l.mlp.kind == MlpConfig::kDense) {
            LK_LAUNCH(launch_gemv_dense(l.up, l.up.mp, in, act, nullptr, kActRelu2, 0, L));
            staged(in.row);
            GemvIn a;
            a.vec = act;
            LK_LAUNCH(launch_gemv_dense(l.down, D, a, y, nullptr, kActNone, 0, L));
        } else {
            LK_LAUNCH(launch_gemv_routed_up(l.moe, in, d_token, act, L));
            staged(in.row);
            LK_LAUNCH(launch_gemv_routed_down(l.moe, D, act, d_token, y, L));
        }
        pending = y, post = l.norm2b;
    }
    if (mode == kStepNoHead) return WICK_ROCM_OK;
    GemvIn in;
    in.row = stage(final_norm), in.row.x_out = nullptr;
    LK_LAUNCH(launch_gemv_dense(head, cfg.vocab, in, logits, nullptr, kActNone, 0, L));
    if (mode == kStepGreedy)
        LK_LAUNCH(launch_argmax(logits, cfg.vocab, d_partial, d_pick, d_token, d_pos, d_history, info.max_seq_len, L, reinterpret_cast<const uint8_t*>(embed),
                                kTypeBF16, cfg.vocab, D, x0));
    return WICK_ROCM_OK;
}

int Lokinex::generate(wick_rocm_ctx* ctx, uint32_t token, uint32_t pos, uint32_t n, uint32_t* out) {
    LK_TRY(set_step(ctx, token, pos));
    for (uint32_t i = 0; i < n; i++) LK_TRY(run_step(ctx, kStepGreedy));
    return wick_rocm_download(ctx, out, d_history + pos, (size_t)n * sizeof(uint32_t));
}

// ---- prompt passes ------------------------------------------------------------------------------------------------------------

int Lokinex::alloc_rows(wick_rocm_ctx* ctx) {
    if (cap) return WICK_ROCM_OK;
    bool exact = f32;
    uint32_t proj_w = 4, mixed_w = 4, act_w = 4, acte_w = 4, u_w = 4, q_w = 4, qa_w = 4, top = 1;
    size_t kx_n = 4, vt_n = 4;
    bool moe = false;
    for (const Layer& l : layers) {
        proj_w = std::max(proj_w, l.in.mp), mixed_w = std::max(mixed_w, l.out.kp);
        if (l.mix.recurrent) u_w = std::max(u_w, l.channels);
        else {
            if (!l.dqp) exact = true;
            qa_w = std::max(qa_w, l.shape.heads * l.shape.row());
            q_w = std::max(q_w, l.shape.heads * 2 * l.dqp);
            kx_n = std::max(kx_n, (size_t)kv_pad() * l.kx.mp), vt_n = std::max(vt_n, (size_t)kv_pad() * l.vx.mp);
        }
        if (l.mlp.kind == MlpConfig::kDense) act_w = std::max(act_w, l.up.mp);
        if (l.mlp.kind == MlpConfig::kMoe) {
            moe = true, top = std::max(top, l.moe.top);
            acte_w = std::max(acte_w, l.moe.down.kp), act_w = std::max(act_w, l.moe.shared_down.kp);
        }
    }
    const uint32_t P = std::min(info.max_seq_len, exact ? kChunkExact : kChunkBf16);
    absorb_cap = exact ? P : std::min(P, kAbsorbMax);
    size_t scratch_n = 4;
    for (const Layer& l : layers) {
        if (l.mix.recurrent) scratch_n = std::max(scratch_n, recurrent_scan_scratch_floats(P, l.channels));
        else
            for (uint32_t n = 1; n <= absorb_cap; n++) scratch_n = std::max(scratch_n, latent_attention_scratch_floats(l.shape, n));
    }
    auto act_rows = [&](size_t count, void** out) { return alloc(ctx, count * act_bytes(), out); };
    const size_t n = P;
    LK_TRY(alloc_t(ctx, n, &p_tokens));
    LK_TRY(alloc_t(ctx, n, &p_rows));
    LK_TRY(alloc_t(ctx, n * dp, &p_x0));
    for (float*& x : p_x) LK_TRY(alloc_t(ctx, n * dp, &x));
    LK_TRY(alloc_t(ctx, n * dp, &p_y));
    LK_TRY(alloc_t(ctx, n * proj_w, &p_proj));
    LK_TRY(alloc_t(ctx, n, &p_gate));
    LK_TRY(alloc_t(ctx, n * u_w, &p_u));
    LK_TRY(alloc_t(ctx, n * u_w, &p_a));
    LK_TRY(alloc_t(ctx, n * u_w, &p_b));
    LK_TRY(alloc_t(ctx, (size_t)absorb_cap * qa_w, &p_qa));
    LK_TRY(alloc_t(ctx, scratch_n, &p_scratch));
    LK_TRY(alloc_t(ctx, (size_t)kHeadRows * vp, &p_logits));
    if (cfg.loop_times) LK_TRY(act_rows(n * loop_terms() * dp, &p_loop));
    LK_TRY(act_rows(n * dp, &p_h));
    LK_TRY(act_rows(n * mixed_w, &p_mixed));
    LK_TRY(act_rows(n * act_w, &p_act));
    LK_TRY(act_rows(n * u_w * (f32 ? 1 : 2), &p_ua));
    if (moe) {
        LK_TRY(act_rows(n * top * acte_w, &p_acte));
        LK_TRY(alloc_t(ctx, n * top * dp, &p_ye));
        std::vector<RouteJob> jobs(n_jobs);
        for (Layer& l : layers) {
            if (l.mlp.kind != MlpConfig::kMoe) continue;
            LK_TRY(alloc_t(ctx, n * l.moe.top, &l.entry_token));
            LK_TRY(alloc_t(ctx, n * l.moe.top, &l.slot_of));
            LK_TRY(alloc_t(ctx, 1, &l.n_tiles));
            LK_TRY(alloc_t(ctx, route_max_tiles(P, l.moe.top, l.moe.experts), &l.tiles));
            jobs[l.job] = RouteJob{l.moe.table, l.moe.top, l.moe.experts, l.entry_token, l.slot_of, l.n_tiles, l.tiles};
        }
        LK_TRY(alloc_t(ctx, jobs.size(), &p_jobs));
        LK_TRY(wick_rocm_upload(ctx, p_jobs, jobs.data(), jobs.size() * sizeof(RouteJob)));
    }
    LK_TRY(alloc_t(ctx, n * q_w, &p_q));
    LK_TRY(alloc_t(ctx, kx_n, &p_kx));
    LK_TRY(alloc_t(ctx, vt_n, &p_vt));
    {
        // positions past a portion's end are read as (weightless) values: whatever the buffer holds there has to be finite
        const std::vector<uint16_t> zeros(vt_n, 0);
        LK_TRY(wick_rocm_upload(ctx, p_vt, zeros.data(), vt_n * 2));
    }
    cap = P;
    return WICK_ROCM_OK;
}

int Lokinex::prompt_mixer(wick_rocm_ctx* ctx, const Layer& l, const Run& r, uint32_t n, uint32_t pos0) {
    const Launch L = ctx->launch();
    const GemmIn h{p_h, dp, n, f32};
    if (l.mix.recurrent) {
        const uint32_t C = l.channels, terms = f32 ? 1 : 2;
        LK_LAUNCH(launch_gemm_gelu_split(l.in, h, p_proj, l.in.mp, l.in_bias, C, L));
        RecurrentConv c{};
        c.proj = p_proj, c.ldp = l.in.mp, c.x_at = C, c.channels = C, c.block = l.block, c.taps = l.mix.conv, c.pos0 = pos0;
        c.w = l.conv, c.bias = l.conv_bias, c.ring = r.conv_ring, c.u = p_u, c.ua = p_ua, c.lda = terms * C, c.f32 = f32;
        LK_LAUNCH(launch_recurrent_conv(c, n, L));
        const GateArgs g{l.r_bias, l.i_bias, l.rate, p_u, p_a, p_b, C};
        LK_LAUNCH(launch_gemm_gates(l.gates, GemmIn{p_ua, terms * C, n, f32}, l.mix.blocks, terms * l.block, g, L));
        LK_LAUNCH(launch_recurrent_scan(p_a, p_b, p_proj, l.in.mp, r.state, n, C, pos0, p_mixed, l.out.kp, l.out.kp, f32, p_scratch, L));
    } else {
        LK_LAUNCH(launch_gemm_store(l.in, h, p_proj, l.in.mp, nullptr, L));
        if (l.dqp && n > kAbsorbMax) {
            const uint32_t keys = pos0 + n;
            LK_LAUNCH(launch_latent_rope(l.shape, l.lat, p_proj, l.in.mp, r.cache, p_q, l.dqp, n, pos0, L));
            const GemmIn rows{r.cache, l.shape.row(), keys, false};
            LK_LAUNCH(launch_gemm_convert(l.kx, rows, p_kx, l.kx.mp, false, L));
            LK_LAUNCH(launch_gemm_convert(l.vx, rows, p_vt, kv_pad(), true, L));
            LK_LAUNCH(launch_latent_prefill(l.shape, p_q, p_kx, l.kx.mp, p_vt, kv_pad(), l.dqp, l.dvp, n, pos0, static_cast<uint16_t*>(p_mixed), l.out.kp, l.out.kp, L));
        } else {
            LK_LAUNCH(launch_latent_absorb(l.shape, l.lat, p_proj, l.in.mp, r.cache, p_qa, n, pos0, nullptr, L));
            LK_LAUNCH(launch_latent_attention(l.shape, l.lat, p_qa, r.cache, p_scratch, n, pos0, nullptr, p_mixed, l.out.kp, l.out.kp, f32, L));
        }
    }
    LK_LAUNCH(launch_gemm_store(l.out, GemmIn{p_mixed, l.out.kp, n, f32}, p_y, dp, nullptr, L));
    return WICK_ROCM_OK;
}

int Lokinex::prompt_mlp(wick_rocm_ctx* ctx, const Layer& l, uint32_t n) {
    const Launch L = ctx->launch();
    const GemmIn h{p_h, dp, n, f32};
    if (l.mlp.kind == MlpConfig::kDense) {
        LK_LAUNCH(launch_gemm_relu2(l.up, h, p_act, l.down.kp, L));
        LK_LAUNCH(launch_gemm_store(l.down, GemmIn{p_act, l.down.kp, n, f32}, p_y, dp, nullptr, L));
        return WICK_ROCM_OK;
    }
    const RoutedMlp& m = l.moe;
    Grouping g{l.tiles, l.n_tiles, route_max_tiles(n, m.top, m.experts), l.entry_token};
    LK_LAUNCH(launch_gemm_silu(m.gate_up, h, p_acte, m.down.kp, nullptr, L, g));
    g.gather = nullptr;
    LK_LAUNCH(launch_gemm_store(m.down, GemmIn{p_acte, m.down.kp, n * m.top, f32}, p_ye, dp, nullptr, L, g));
    if (m.shared_gate_up.d) {
        LK_LAUNCH(launch_gemm_silu(m.shared_gate_up, h, p_act, m.shared_down.kp, p_gate, L));
        LK_LAUNCH(launch_gemm_store(m.shared_down, GemmIn{p_act, m.shared_down.kp, n, f32}, p_y, dp, nullptr, L));
    }
    return WICK_ROCM_OK;
}

int Lokinex::prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                         float* layers_out) {
    const Launch L = ctx->launch();
    const uint32_t D = cfg.width;
    LK_TRY(wick_rocm_upload(ctx, p_tokens, tokens, (size_t)n * sizeof(uint32_t)));
    char* x0_at = p_loop ? static_cast<char*>(p_loop) + (size_t)dp * act_bytes() : nullptr;
    LK_LAUNCH(launch_embed_activation(embed, cfg.vocab, D, p_tokens, n, p_x0, dp, x0_at, loop_terms() * dp, dp, f32, L));
    LK_LAUNCH(launch_route(p_jobs, n_jobs, p_tokens, n, L));

    const float* x = p_x0;
    RowStage pend;  // y / experts / slots / top / g_post of the sublayer whose output is still to be added
    auto rows = [&](float g_pre, bool keep) {
        RowsArgs a;
        a.s = pend;
        a.s.x = x, a.s.x_stride = dp, a.s.y_stride = dp, a.s.g_pre = g_pre, a.s.eps = (float)cfg.eps, a.s.dim = D;
        if (keep && (pend.y || pend.experts)) a.s.x_out = x == p_x[0] ? p_x[1] : p_x[0];
        a.n = n, a.pos0 = pos0, a.out = p_h, a.ldo = dp, a.kp = dp, a.f32 = f32;
        return a;
    };
    auto done = [&](const RowsArgs& a) {
        if (a.s.x_out) x = a.s.x_out;
        pend = RowStage();
    };
    for (uint32_t i = 0; i < runs.size(); i++) {
        const Run& r = runs[i];
        const Layer& l = layers[r.layer];
        if (r.pass >= 0) {
            RowsArgs a = rows(0.0f, false);
            a.out = p_loop, a.ldo = loop_terms() * dp, a.lo_at = 2 * dp;
            LK_LAUNCH(launch_rows(a, kRowSplit, L));
            float* out = x == p_x[0] ? p_x[1] : p_x[0];
            LK_LAUNCH(launch_gemm_store(loop_in, GemmIn{p_loop, loop_terms() * dp, n, f32}, out, dp, loop_step + (size_t)r.pass * dp, L));
            x = out, pend = RowStage();
        }
        {
            RowsArgs a = rows(l.norm1, true);
            a.s.conv = l.canon, a.s.ring = r.canon_ring, a.s.taps = cfg.taps;
            LK_LAUNCH(launch_rows(a, kRowNorm, L));
            done(a);
        }
        LK_TRY(prompt_mixer(ctx, l, r, n, pos0));
        pend.y = p_y, pend.g_post = l.norm1b;
        if (l.mlp.kind != MlpConfig::kNone) {
            RowsArgs a = rows(l.norm2, true);
            if (l.moe.shared_sg) a.gate_w = l.moe.shared_sg, a.row_gate = p_gate;
            LK_LAUNCH(launch_rows(a, kRowNorm, L));
            done(a);
            LK_TRY(prompt_mlp(ctx, l, n));
            pend.g_post = l.norm2b;
            if (l.mlp.kind == MlpConfig::kMoe) {
                pend.experts = p_ye, pend.slots = l.slot_of, pend.top = l.moe.top;
                if (l.moe.shared_gate_up.d) pend.y = p_y;
            } else {
                pend.y = p_y;
            }
        }
        if (layers_out) {
            if (!p_trace) LK_TRY(alloc_t(ctx, (size_t)cap * dp, &p_trace));
            RowsArgs a = rows(0.0f, false);
            a.s.x_out = p_trace;
            LK_LAUNCH(launch_rows(a, kRowOnly, L));
            std::vector<float> host((size_t)n * dp);
            LK_TRY(wick_rocm_download(ctx, host.data(), p_trace, host.size() * sizeof(float)));
            for (uint32_t t = 0; t < n; t++) memcpy(layers_out + ((size_t)i * n + t) * D, &host[(size_t)t * dp], (size_t)D * sizeof(float));
        }
    }
    if (n_want == 0) return WICK_ROCM_OK;
    LK_TRY(wick_rocm_upload(ctx, p_rows, want, (size_t)n_want * sizeof(uint32_t)));
    if (n_want <= kHeadGemvRows) {
        RowsArgs a = rows(0.0f, true);
        a.n = n_want, a.rows = p_rows;
        if (a.s.x_out) {  // the wanted rows of the finished residual
            LK_LAUNCH(launch_rows(a, kRowOnly, L));
            x = a.s.x_out;
        }
        for (uint32_t i = 0; i < n_want; i++) {
            GemvIn in;
            in.row.x = x + (size_t)want[i] * dp, in.row.x_stride = dp, in.row.g_pre = final_norm, in.row.eps = (float)cfg.eps, in.row.dim = D;
            LK_LAUNCH(launch_gemv_dense(head, cfg.vocab, in, p_logits + (size_t)i * vp, nullptr, kActNone, 0, L));
        }
        for (uint32_t i = 0; i < n_want; i++)
            LK_TRY(wick_rocm_download(ctx, logits_out + (size_t)i * cfg.vocab, p_logits + (size_t)i * vp, (size_t)cfg.vocab * sizeof(float)));
        return WICK_ROCM_OK;
    }
    std::vector<float> host;
    for (uint32_t first = 0; first < n_want; first += kHeadRows) {
        const uint32_t count = std::min(kHeadRows, n_want - first);
        RowsArgs a = rows(final_norm, false);
        a.n = count, a.rows = p_rows + first;
        LK_LAUNCH(launch_rows(a, kRowNorm, L));
        LK_LAUNCH(launch_gemm_store(head, GemmIn{p_h, dp, count, f32}, p_logits, vp, nullptr, L));
        host.resize((size_t)count * vp);
        LK_TRY(wick_rocm_download(ctx, host.data(), p_logits, host.size() * sizeof(float)));
        for (uint32_t i = 0; i < count; i++)
            memcpy(logits_out + (size_t)(first + i) * cfg.vocab, &host[(size_t)i * vp], (size_t)cfg.vocab * sizeof(float));
    }
    return WICK_ROCM_OK;
}

int Lokinex::forward(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos, const uint32_t* want, uint32_t n_want, float* logits_out,
                     float* layers_out) {
    if (n <= kStepsMax && !layers_out) {
        uint32_t w = 0;
        for (uint32_t i = 0; i < n; i++) {
            const bool wanted = w < n_want && want[w] == i;
            LK_TRY(set_step(ctx, tokens[i], pos + i));
            LK_TRY(run_step(ctx, wanted ? kStepLogits : kStepNoHead));
            if (wanted) LK_TRY(wick_rocm_download(ctx, logits_out + (size_t)w++ * cfg.vocab, logits, (size_t)cfg.vocab * sizeof(float)));
        }
        return wick_rocm_sync(ctx);
    }
    LK_TRY(alloc_rows(ctx));
    if (layers_out && n > cap) return ctx_fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "per-layer copies: more tokens than one prompt pass takes");
    uint32_t w = 0;
    for (uint32_t at = 0; at < n; at += cap) {
        const uint32_t count = std::min(cap, n - at);
        std::vector<uint32_t> here;
        const uint32_t w0 = w;
        while (w < n_want && want[w] < at + count) here.push_back(want[w++] - at);
        LK_TRY(prompt_pass(ctx, tokens + at, count, pos + at, here.data(), (uint32_t)here.size(), logits_out + (size_t)w0 * cfg.vocab, layers_out));
    }
    return wick_rocm_sync(ctx);
}

// ---- state --------------------------------------------------------------------------------------------------------------------

template <typename F>
int Lokinex::for_each_state_piece(uint32_t seq_len, F&& piece) const {
    for (const Run& r : runs) {
        const Layer& l = layers[r.layer];
        LK_TRY(piece(r.canon_ring, (size_t)cfg.taps * dp * sizeof(float)));
        if (l.mix.recurrent) {
            LK_TRY(piece(r.conv_ring, (size_t)l.mix.conv * l.channels * sizeof(float)));
            LK_TRY(piece(r.state, (size_t)l.channels * sizeof(float)));
        } else if (seq_len) {
            LK_TRY(piece(r.cache, (size_t)seq_len * l.shape.row() * act_bytes()));
        }
    }
    return WICK_ROCM_OK;
}

size_t Lokinex::state_bytes(uint32_t seq_len) const {
    size_t total = 0;
    for_each_state_piece(seq_len, [&](const void*, size_t n) {
        total += n;
        return WICK_ROCM_OK;
    });
    return total;
}

int Lokinex::snapshot(wick_rocm_ctx* ctx, uint32_t seq_len, void* out) {
    char* at = static_cast<char*>(out);
    return for_each_state_piece(seq_len, [&](const void* d, size_t n) {
        const int rc = wick_rocm_download(ctx, at, d, n);
        at += n;
        return rc;
    });
}

int Lokinex::restore(wick_rocm_ctx* ctx, uint32_t seq_len, const void* in) {
    const char* at = static_cast<const char*>(in);
    return for_each_state_piece(seq_len, [&](void* d, size_t n) {
        const int rc = wick_rocm_upload(ctx, d, at, n);
        at += n;
        return rc;
    });
}

}  // namespace

int load_lokinex(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out) {
    std::unique_ptr<Lokinex> m(new Lokinex);
    m->f32 = dtype == WICK_ROCM_MODEL_F32;
    int rc;
    try {
        rc = m->load(ctx, folder, context_size);
    } catch (const ConfigError& e) {
        rc = ctx_fail(ctx, WICK_ROCM_ERR_BAD_SHAPE, e.what);
    }
    if (rc) {
        m->release(ctx);
        return rc;
    }
    *out = m.release();
    return WICK_ROCM_OK;
}
