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
#include "folder_model.h"

namespace {

using namespace folder_model;

constexpr uint32_t kChunkBf16 = 2048, kChunkExact = 512;  // tokens per prompt pass: bfloat16 / f32 or a head shape without matrix-core attention
constexpr uint32_t kAbsorbMax = 16;     // portions this short attend with absorbed queries, without expanding the cache

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

struct Lokinex final : FolderModel {
    Config cfg;
    DenseWeight loop_in;
    float* loop_step = nullptr; // [times][dp]
    std::vector<Layer> layers;
    std::vector<Run> runs;
    // a step's vectors
    float *y = nullptr, *proj = nullptr, *mixed = nullptr, *act = nullptr, *qa = nullptr, *scratch = nullptr;
    // a prompt pass's rows
    float *p_y = nullptr, *p_ye = nullptr, *p_proj = nullptr, *p_gate = nullptr, *p_u = nullptr, *p_a = nullptr, *p_b = nullptr, *p_qa = nullptr,
          *p_scratch = nullptr;
    void *p_loop = nullptr, *p_mixed = nullptr, *p_act = nullptr, *p_acte = nullptr, *p_ua = nullptr;
    uint16_t *p_q = nullptr, *p_kx = nullptr, *p_vt = nullptr;
    RouteJob* p_jobs = nullptr;
    uint32_t n_jobs = 0, absorb_cap = 0;

    uint32_t loop_terms() const { return f32 ? 2 : 3; }  // columns of the loop's input in units of dp: x (hi) | x0 (| x lo)
    uint32_t kv_pad() const { return pad_to(info.max_seq_len, 64); }

    int load(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t context_size);
    int load_layer(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t i);
    int enqueue_step(wick_rocm_ctx* ctx, StepMode mode) override;
    int alloc_rows(wick_rocm_ctx* ctx) override;
    int prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                    float* layers_out) override;
    int prompt_mixer(wick_rocm_ctx* ctx, const Layer& l, const Run& r, uint32_t n, uint32_t pos0);
    int prompt_mlp(wick_rocm_ctx* ctx, const Layer& l, uint32_t n);
    std::vector<StatePiece> state_pieces(uint32_t seq_len) const override;
};

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

// ---- weights ----------------------------------------------------------------------------------------------------------------

int Lokinex::load_layer(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t i) {
    const std::string p = "l" + std::to_string(i) + ".", mp = p + "mix.", fp = p + "mlp.";
    Layer& l = layers[i];
    const uint32_t D = cfg.width;
    const MixerConfig& m = l.mix = cfg.layers[i].first;
    const MlpConfig& c = l.mlp = cfg.layers[i].second;
    l.norm1 = scalar(f, p + "norm1"), l.norm1b = scalar(f, p + "norm1b");
    MODEL_TRY(upload(ctx, taps_by_time(tensor(f, p + "canon1", {D, cfg.taps}), D, cfg.taps, dp, [](uint32_t e) { return e; }), &l.canon));
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
            MODEL_TRY(upload(ctx, w, &l.in));
            std::vector<float> b = spread(tensor(f, mp + "y.b", {W})), bx = spread(tensor(f, mp + "x.b", {W}));
            b.insert(b.end(), bx.begin(), bx.end());
            MODEL_TRY(upload(ctx, b, &l.in_bias));
        }
        MODEL_TRY(upload(ctx, taps_by_time(tensor(f, mp + "conv", {W, m.conv}), W, m.conv, C, at), &l.conv));
        MODEL_TRY(upload(ctx, spread(tensor(f, mp + "conv.b", {W})), &l.conv_bias));
        {
            // bfloat16 products take u as two terms: the block's columns once per term
            const uint32_t terms = f32 ? 1 : 2;
            Packer w(m.blocks, 2 * bp, terms * bp);
            const uint16_t *ra = tensor(f, mp + "ra", {m.blocks, bs, bs}), *ri = tensor(f, mp + "ri", {m.blocks, bs, bs});
            for (uint32_t b = 0; b < m.blocks; b++)
                for (uint32_t t = 0; t < terms; t++) w.pair(b, ra + (size_t)b * bs * bs, ri + (size_t)b * bs * bs, bs, bs, t * bp);
            MODEL_TRY(upload(ctx, w, &l.gates));
            MODEL_TRY(upload(ctx, spread(tensor(f, mp + "ra.b", {m.blocks, bs})), &l.r_bias));
            MODEL_TRY(upload(ctx, spread(tensor(f, mp + "ri.b", {m.blocks, bs})), &l.i_bias));
            std::vector<float> rate(C, 0.0f);
            const uint16_t* lam = tensor(f, mp + "lam", {W});
            for (uint32_t ch = 0; ch < W; ch++) {
                const double z = bf16(lam[ch]);
                rate[at(ch)] = (float)(-8.0 * (std::fmax(z, 0.0) + std::log1p(std::exp(-std::fabs(z)))));  // -8 softplus(lam)
            }
            MODEL_TRY(upload(ctx, rate, &l.rate));
        }
        Packer o(1, D, C);
        const uint16_t* wo = tensor(f, mp + "o", {D, W});
        for (uint32_t r = 0; r < D; r++)
            for (uint32_t b = 0; b < m.blocks; b++) o.row(0, r, wo + (size_t)r * W + b * bs, bs, b * bp);
        MODEL_TRY(upload(ctx, o, &l.out));
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
        MODEL_TRY(upload(ctx, w, &l.in));
        const uint16_t *uk = tensor(f, mp + "uk", {H * m.dim, m.rank}), *uv = tensor(f, mp + "uv", {H * m.vdim, m.rank});
        auto padded = [&](const uint16_t* src, uint32_t rows) {
            std::vector<uint16_t> v((size_t)rows * s.rank_p, 0);
            for (uint32_t r = 0; r < rows; r++) memcpy(&v[(size_t)r * s.rank_p], src + (size_t)r * m.rank, (size_t)m.rank * 2);
            return v;
        };
        uint16_t *d_uk = nullptr, *d_uv = nullptr;
        MODEL_TRY(upload(ctx, padded(uk, H * m.dim), &d_uk));
        MODEL_TRY(upload(ctx, padded(uv, H * m.vdim), &d_uv));
        float *d_norm = nullptr, *rope = nullptr;
        MODEL_TRY(upload(ctx, widened(tensor(f, mp + "dkv.norm", {m.rank}), m.rank), &d_norm));
        MODEL_TRY(upload_rope(ctx, rope_frequencies(m.rope_base, m.rot), &rope));
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
            MODEL_TRY(upload(ctx, k, &l.kx));
            MODEL_TRY(upload(ctx, v, &l.vx));
        } else {
            l.dqp = l.dvp = 0;
        }
        Packer o(1, D, H * m.vdim);
        o.rows(0, 0, tensor(f, mp + "o", {D, H * m.vdim}), D, H * m.vdim);
        MODEL_TRY(upload(ctx, o, &l.out));
    }
    if (c.kind == MlpConfig::kNone) return WICK_ROCM_OK;
    l.norm2 = scalar(f, p + "norm2"), l.norm2b = scalar(f, p + "norm2b");
    if (c.kind == MlpConfig::kDense) {
        Packer up(1, c.ff, D), down(1, D, c.ff);
        up.rows(0, 0, tensor(f, fp + "up", {c.ff, D}), c.ff, D);
        down.rows(0, 0, tensor(f, fp + "down", {D, c.ff}), D, c.ff);
        MODEL_TRY(upload(ctx, up, &l.up));
        return upload(ctx, down, &l.down);
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
        MODEL_TRY(upload(ctx, gu, &r.gate_up));
        MODEL_TRY(upload(ctx, down, &r.down));
    }
    if (c.shared_ff) {
        Packer gu(1, 2 * pad_to(c.shared_ff, kDensePad), D), down(1, D, c.shared_ff), sg(1, 1, D);
        gu.pair(0, tensor(f, fp + "shared.gate", {c.shared_ff, D}), tensor(f, fp + "shared.up", {c.shared_ff, D}), c.shared_ff, D);
        down.rows(0, 0, tensor(f, fp + "shared.down", {D, c.shared_ff}), D, c.shared_ff);
        sg.row(0, 0, tensor(f, fp + "shared.sg", {1, D}), D);
        DenseWeight w;
        MODEL_TRY(upload(ctx, gu, &r.shared_gate_up));
        MODEL_TRY(upload(ctx, down, &r.shared_down));
        MODEL_TRY(upload(ctx, sg, &w));
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
    MODEL_TRY(alloc_t(ctx, table.size(), &d_table));
    MODEL_TRY(wick_rocm_upload(ctx, d_table, table.data(), table.size() * 4));
    r.table = d_table;
    l.job = n_jobs++;
    return WICK_ROCM_OK;
}

int Lokinex::load(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t context_size) {
    cfg = read_config(f->config);
    const uint32_t D = cfg.width;
    eps = (float)cfg.eps;
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

    MODEL_TRY(load_ends(ctx, f, "Lokinex", cfg.vocab, D, context_size, "head"));
    final_norm.g = scalar(f, "final.norm");
    if (cfg.loop_times) {
        // [x | x0], and for bfloat16 products the low term of x behind them over the same columns of the weight
        Packer w(1, D, loop_terms() * dp);
        const uint16_t* src = tensor(f, "loop.in", {D, 2 * D});
        for (uint32_t r = 0; r < D; r++) {
            w.row(0, r, src + (size_t)r * 2 * D, D, 0), w.row(0, r, src + (size_t)r * 2 * D + D, D, dp);
            if (!f32) w.row(0, r, src + (size_t)r * 2 * D, D, 2 * dp);
        }
        MODEL_TRY(upload(ctx, w, &loop_in));
        const uint16_t* st = tensor(f, "loop.step", {cfg.loop_times, D});
        std::vector<float> v((size_t)cfg.loop_times * dp, 0.0f);
        for (uint32_t t = 0; t < cfg.loop_times; t++)
            for (uint32_t k = 0; k < D; k++) v[(size_t)t * dp + k] = bf16(st[(size_t)t * D + k]);
        MODEL_TRY(upload(ctx, v, &loop_step));
    }
    layers.resize(cfg.layers.size());
    for (uint32_t i = 0; i < layers.size(); i++) MODEL_TRY(load_layer(ctx, f, i));

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
        MODEL_TRY(alloc_t(ctx, (size_t)cfg.taps * dp, &r.canon_ring));
        proj_w = std::max(proj_w, l.in.mp), mixed_w = std::max(mixed_w, l.out.kp);
        if (l.mix.recurrent) {
            MODEL_TRY(alloc_t(ctx, (size_t)l.mix.conv * l.channels, &r.conv_ring));
            MODEL_TRY(alloc_t(ctx, l.channels, &r.state));
        } else {
            MODEL_TRY(alloc(ctx, (size_t)info.max_seq_len * l.shape.row() * act_bytes(), &r.cache));
            qa_w = std::max(qa_w, l.shape.heads * l.shape.row());
            scratch_w = std::max(scratch_w, latent_attention_scratch_floats(l.shape, 1));
        }
        if (l.mlp.kind == MlpConfig::kDense) act_w = std::max(act_w, l.up.mp);
        if (l.mlp.kind == MlpConfig::kMoe) act_w = std::max(act_w, routed_act_floats(l.moe));
    }
    MODEL_TRY(alloc_step(ctx));
    MODEL_TRY(alloc_t(ctx, dp, &y));
    MODEL_TRY(alloc_t(ctx, proj_w, &proj));
    MODEL_TRY(alloc_t(ctx, mixed_w, &mixed));
    MODEL_TRY(alloc_t(ctx, act_w, &act));
    MODEL_TRY(alloc_t(ctx, qa_w, &qa));
    MODEL_TRY(alloc_t(ctx, scratch_w, &scratch));
    return wick_rocm_sync(ctx);
}

// ---- one step ----------------------------------------------------------------------------------------------------------------

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
        s.x = x, s.x_stride = dp, s.y = pending, s.y_stride = dp, s.g_post = post, s.g_pre = g_pre, s.eps = eps, s.dim = D;
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
            MODEL_LAUNCH(launch_gemv_dense(loop_in, D, in, out, loop_step + (size_t)r.pass * dp, kActNone, 0, L));
            x = out, pending = nullptr;
        }
        {
            GemvIn in;
            in.row = stage(l.norm1), in.d_pos = d_pos;
            in.row.conv = l.canon, in.row.ring = r.canon_ring, in.row.taps = cfg.taps;
            MODEL_LAUNCH(launch_gemv_dense(l.in, l.in.mp, in, proj, l.mix.recurrent ? l.in_bias : nullptr, l.mix.recurrent ? kActGeluSplit : kActNone, l.channels, L));
            staged(in.row);
        }
        if (l.mix.recurrent) {
            RecurrentStep s{};
            s.proj = proj, s.channels = l.channels, s.block = l.block, s.blocks = l.mix.blocks, s.taps = l.mix.conv;
            s.conv_w = l.conv, s.conv_bias = l.conv_bias, s.ring = r.conv_ring, s.state = r.state, s.gates = l.gates;
            s.r_bias = l.r_bias, s.i_bias = l.i_bias, s.rate = l.rate, s.out = mixed, s.d_pos = d_pos;
            MODEL_LAUNCH(launch_recurrent_step(s, L));
        } else {
            MODEL_LAUNCH(launch_latent_absorb(l.shape, l.lat, proj, l.in.mp, r.cache, qa, 1, 0, d_pos, L));
            MODEL_LAUNCH(launch_latent_attention(l.shape, l.lat, qa, r.cache, scratch, 1, 0, d_pos, mixed, l.out.kp, l.out.kp, true, L));
        }
        GemvIn mix;
        mix.vec = mixed;
        MODEL_LAUNCH(launch_gemv_dense(l.out, D, mix, y, nullptr, kActNone, 0, L));
        pending = y, post = l.norm1b;
        if (l.mlp.kind == MlpConfig::kNone) continue;
        GemvIn in;
        in.row = stage(l.norm2);
        if (l.mlp.kind == MlpConfig::kDense) {
            MODEL_LAUNCH(launch_gemv_dense(l.up, l.up.mp, in, act, nullptr, kActRelu2, 0, L));
            staged(in.row);
            GemvIn a;
            a.vec = act;
            MODEL_LAUNCH(launch_gemv_dense(l.down, D, a, y, nullptr, kActNone, 0, L));
        } else {
            MODEL_LAUNCH(launch_gemv_routed_up(l.moe, in, d_token, act, L));
            staged(in.row);
            MODEL_LAUNCH(launch_gemv_routed_down(l.moe, D, act, d_token, y, L));
        }
        pending = y, post = l.norm2b;
    }
    GemvIn in;
    in.row = stage(final_norm.g), in.row.x_out = nullptr;
    return finish_step(ctx, mode, in);
}

// ---- prompt passes ------------------------------------------------------------------------------------------------------------

int Lokinex::alloc_rows(wick_rocm_ctx* ctx) {
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
    const size_t n = P;
    MODEL_TRY(alloc_pass(ctx, P));
    MODEL_TRY(alloc_t(ctx, n * dp, &p_y));
    MODEL_TRY(alloc_t(ctx, n * proj_w, &p_proj));
    MODEL_TRY(alloc_t(ctx, n, &p_gate));
    MODEL_TRY(alloc_t(ctx, n * u_w, &p_u));
    MODEL_TRY(alloc_t(ctx, n * u_w, &p_a));
    MODEL_TRY(alloc_t(ctx, n * u_w, &p_b));
    MODEL_TRY(alloc_t(ctx, (size_t)absorb_cap * qa_w, &p_qa));
    MODEL_TRY(alloc_t(ctx, scratch_n, &p_scratch));
    if (cfg.loop_times) MODEL_TRY(alloc_act(ctx, n * loop_terms() * dp, &p_loop));
    MODEL_TRY(alloc_act(ctx, n * mixed_w, &p_mixed));
    MODEL_TRY(alloc_act(ctx, n * act_w, &p_act));
    MODEL_TRY(alloc_act(ctx, n * u_w * (f32 ? 1 : 2), &p_ua));
    if (moe) {
        MODEL_TRY(alloc_act(ctx, n * top * acte_w, &p_acte));
        MODEL_TRY(alloc_t(ctx, n * top * dp, &p_ye));
        std::vector<RouteJob> jobs(n_jobs);
        for (Layer& l : layers) {
            if (l.mlp.kind != MlpConfig::kMoe) continue;
            MODEL_TRY(alloc_t(ctx, n * l.moe.top, &l.entry_token));
            MODEL_TRY(alloc_t(ctx, n * l.moe.top, &l.slot_of));
            MODEL_TRY(alloc_t(ctx, 1, &l.n_tiles));
            MODEL_TRY(alloc_t(ctx, route_max_tiles(P, l.moe.top, l.moe.experts), &l.tiles));
            jobs[l.job] = RouteJob{l.moe.table, l.moe.top, l.moe.experts, l.entry_token, l.slot_of, l.n_tiles, l.tiles};
        }
        MODEL_TRY(alloc_t(ctx, jobs.size(), &p_jobs));
        MODEL_TRY(wick_rocm_upload(ctx, p_jobs, jobs.data(), jobs.size() * sizeof(RouteJob)));
    }
    MODEL_TRY(alloc_t(ctx, n * q_w, &p_q));
    MODEL_TRY(alloc_t(ctx, kx_n, &p_kx));
    MODEL_TRY(alloc_t(ctx, vt_n, &p_vt));
    {
        // positions past a portion's end are read as (weightless) values: whatever the buffer holds there has to be finite
        const std::vector<uint16_t> zeros(vt_n, 0);
        MODEL_TRY(wick_rocm_upload(ctx, p_vt, zeros.data(), vt_n * 2));
    }
    cap = P;
    return WICK_ROCM_OK;
}

int Lokinex::prompt_mixer(wick_rocm_ctx* ctx, const Layer& l, const Run& r, uint32_t n, uint32_t pos0) {
    const Launch L = ctx->launch();
    const GemmIn h{p_h, dp, n, f32};
    if (l.mix.recurrent) {
        const uint32_t C = l.channels, terms = f32 ? 1 : 2;
        MODEL_LAUNCH(launch_gemm_gelu_split(l.in, h, p_proj, l.in.mp, l.in_bias, C, L));
        RecurrentConv c{};
        c.proj = p_proj, c.ldp = l.in.mp, c.x_at = C, c.channels = C, c.block = l.block, c.taps = l.mix.conv, c.pos0 = pos0;
        c.w = l.conv, c.bias = l.conv_bias, c.ring = r.conv_ring, c.u = p_u, c.ua = p_ua, c.lda = terms * C, c.f32 = f32;
        MODEL_LAUNCH(launch_recurrent_conv(c, n, L));
        const GateArgs g{l.r_bias, l.i_bias, l.rate, p_u, p_a, p_b, C};
        MODEL_LAUNCH(launch_gemm_gates(l.gates, GemmIn{p_ua, terms * C, n, f32}, l.mix.blocks, terms * l.block, g, L));
        MODEL_LAUNCH(launch_recurrent_scan(p_a, p_b, p_proj, l.in.mp, r.state, n, C, pos0, p_mixed, l.out.kp, l.out.kp, f32, p_scratch, L));
    } else {
        MODEL_LAUNCH(launch_gemm_store(l.in, h, p_proj, l.in.mp, nullptr, L));
        if (l.dqp && n > kAbsorbMax) {
            const uint32_t keys = pos0 + n;
            MODEL_LAUNCH(launch_latent_rope(l.shape, l.lat, p_proj, l.in.mp, r.cache, p_q, l.dqp, n, pos0, L));
            const GemmIn rows{r.cache, l.shape.row(), keys, false};
            MODEL_LAUNCH(launch_gemm_convert(l.kx, rows, p_kx, l.kx.mp, false, L));
            MODEL_LAUNCH(launch_gemm_convert(l.vx, rows, p_vt, kv_pad(), true, L));
            MODEL_LAUNCH(launch_latent_prefill(l.shape, p_q, p_kx, l.kx.mp, p_vt, kv_pad(), l.dqp, l.dvp, n, pos0, static_cast<uint16_t*>(p_mixed), l.out.kp, l.out.kp, L));
        } else {
            MODEL_LAUNCH(launch_latent_absorb(l.shape, l.lat, p_proj, l.in.mp, r.cache, p_qa, n, pos0, nullptr, L));
            MODEL_LAUNCH(launch_latent_attention(l.shape, l.lat, p_qa, r.cache, p_scratch, n, pos0, nullptr, p_mixed, l.out.kp, l.out.kp, f32, L));
        }
    }
    MODEL_LAUNCH(launch_gemm_store(l.out, GemmIn{p_mixed, l.out.kp, n, f32}, p_y, dp, nullptr, L));
    return WICK_ROCM_OK;
}

int Lokinex::prompt_mlp(wick_rocm_ctx* ctx, const Layer& l, uint32_t n) {
    const Launch L = ctx->launch();
    const GemmIn h{p_h, dp, n, f32};
    if (l.mlp.kind == MlpConfig::kDense) {
        MODEL_LAUNCH(launch_gemm_relu2(l.up, h, p_act, l.down.kp, L));
        MODEL_LAUNCH(launch_gemm_store(l.down, GemmIn{p_act, l.down.kp, n, f32}, p_y, dp, nullptr, L));
        return WICK_ROCM_OK;
    }
    const RoutedMlp& m = l.moe;
    Grouping g{l.tiles, l.n_tiles, route_max_tiles(n, m.top, m.experts), l.entry_token};
    MODEL_LAUNCH(launch_gemm_silu(m.gate_up, h, p_acte, m.down.kp, nullptr, L, g));
    g.gather = nullptr;
    MODEL_LAUNCH(launch_gemm_store(m.down, GemmIn{p_acte, m.down.kp, n * m.top, f32}, p_ye, dp, nullptr, L, g));
    if (m.shared_gate_up.d) {
        MODEL_LAUNCH(launch_gemm_silu(m.shared_gate_up, h, p_act, m.shared_down.kp, p_gate, L));
        MODEL_LAUNCH(launch_gemm_store(m.shared_down, GemmIn{p_act, m.shared_down.kp, n, f32}, p_y, dp, nullptr, L));
    }
    return WICK_ROCM_OK;
}

int Lokinex::prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                         float* layers_out) {
    const Launch L = ctx->launch();
    const uint32_t D = cfg.width;
    MODEL_TRY(wick_rocm_upload(ctx, p_tokens, tokens, (size_t)n * sizeof(uint32_t)));
    char* x0_at = p_loop ? static_cast<char*>(p_loop) + (size_t)dp * act_bytes() : nullptr;
    MODEL_LAUNCH(launch_embed_activation(embed, cfg.vocab, D, embed_scale, p_tokens, n, p_x0, dp, x0_at, loop_terms() * dp, dp, f32, L));
    MODEL_LAUNCH(launch_route(p_jobs, n_jobs, p_tokens, n, L));

    const float* x = p_x0;
    RowStage pend;  // y / experts / slots / top / g_post of the sublayer whose output is still to be added
    auto rows = [&](float g_pre, bool keep) { return rows_of(pend, x, Gain{g_pre, nullptr}, keep, n, pos0); };
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
            MODEL_LAUNCH(launch_rows(a, kRowSplit, L));
            float* out = x == p_x[0] ? p_x[1] : p_x[0];
            MODEL_LAUNCH(launch_gemm_store(loop_in, GemmIn{p_loop, loop_terms() * dp, n, f32}, out, dp, loop_step + (size_t)r.pass * dp, L));
            x = out, pend = RowStage();
        }
        {
            RowsArgs a = rows(l.norm1, true);
            a.s.conv = l.canon, a.s.ring = r.canon_ring, a.s.taps = cfg.taps;
            MODEL_LAUNCH(launch_rows(a, kRowNorm, L));
            done(a);
        }
        MODEL_TRY(prompt_mixer(ctx, l, r, n, pos0));
        pend.y = p_y, pend.g_post = l.norm1b;
        if (l.mlp.kind != MlpConfig::kNone) {
            RowsArgs a = rows(l.norm2, true);
            if (l.moe.shared_sg) a.gate_w = l.moe.shared_sg, a.row_gate = p_gate;
            MODEL_LAUNCH(launch_rows(a, kRowNorm, L));
            done(a);
            MODEL_TRY(prompt_mlp(ctx, l, n));
            pend.g_post = l.norm2b;
            if (l.mlp.kind == MlpConfig::kMoe) {
                pend.experts = p_ye, pend.slots = l.slot_of, pend.top = l.moe.top;
                if (l.moe.shared_gate_up.d) pend.y = p_y;
            } else {
                pend.y = p_y;
            }
        }
        if (layers_out) MODEL_TRY(copy_residual(ctx, pend, x, n, layers_out + (size_t)i * n * D));
    }
    return wanted_logits(ctx, pend, x, want, n_want, logits_out);
}

// ---- state --------------------------------------------------------------------------------------------------------------------

std::vector<StatePiece> Lokinex::state_pieces(uint32_t seq_len) const {
    std::vector<StatePiece> v;
    for (const Run& r : runs) {
        const Layer& l = layers[r.layer];
        v.push_back({r.canon_ring, (size_t)cfg.taps * dp * sizeof(float)});
        if (l.mix.recurrent) {
            v.push_back({r.conv_ring, (size_t)l.mix.conv * l.channels * sizeof(float)});
            v.push_back({r.state, (size_t)l.channels * sizeof(float)});
        } else if (seq_len) {
            v.push_back({r.cache, (size_t)seq_len * l.shape.row() * act_bytes()});
        }
    }
    return v;
}

}  // namespace

int load_lokinex(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out) {
    return load_folder_model<Lokinex>(ctx, folder, dtype, context_size, out);
}
