// The Zirurax model: config.json and tensors of a model folder -> packed weights, caches and states -> steps and prompt passes over the
// kernels of wick_rocm_dense.h.  Host code only.
//
// A decoder whose layers add three sublayers of one norm at once: grouped-query attention over a sliding window (partial rotary positions,
// capped scores, gated output) and a state-space duality block, their outputs normed and averaged, and a dense feed-forward.  All their
// projections of the norm are one product.
//
// State of a sequence, per layer: a ring of keys and values that holds a window and a prompt pass, the ring of the convolution's last
// inputs, the recurrent state.  Rings are addressed by position and a recurrent state is only read past position 0, so a sequence that
// starts at position 0 needs nothing cleared.
#include "folder_model.h"

namespace {

using namespace folder_model;

constexpr uint32_t kChunkBf16 = 2048, kChunkExact = 512;  // tokens per prompt pass: bfloat16 / f32 or heads without matrix-core attention
constexpr uint32_t kShortMax = 16;                        // portions this short run token by token through attention and state
constexpr uint32_t kForkMin = 256;                        // longer portions run attention and state side by side

struct AttentionConfig {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, window = 0, rot = 0;
    double scale = 0.0, softcap = 0.0;
    std::vector<double> freqs;
};
struct SsdConfig {
    uint32_t heads = 0, groups = 0, state = 0, vdim = 0, conv = 0, parts = 0;
};
struct LayerConfig {
    AttentionConfig left;
    SsdConfig right;
    uint32_t ff = 0;  // 0: no feed-forward
};
struct Config {
    uint32_t vocab = 0, width = 0;
    double eps = 0.0, embed_scale = 1.0;
    std::vector<LayerConfig> layers;
};

struct Layer {
    LayerConfig c;
    float *norm = nullptr, *left_gain = nullptr, *right_gain = nullptr;
    DenseWeight in, left_out, right_out, down;
    uint32_t split = 0;  // rows of `in` in front of the feed-forward's pairs
    // where the projection's columns start
    uint32_t q_at = 0, k_at = 0, v_at = 0, g_at = 0, z_at = 0, x_at = 0, dt_at = 0;
    WindowShape window{};
    float* rope = nullptr;
    SsdShape ssd{};
    SsdWeights ssd_w{};
    float* ssd_norm = nullptr;
    // state of the sequence
    void *keys = nullptr, *values = nullptr;
    float *ring = nullptr, *state = nullptr;

    uint32_t inner() const { return c.right.heads * c.right.vdim; }
    WindowProj window_proj(const float* p) const { return WindowProj{p, split, q_at, k_at, v_at, g_at, rope}; }
    SsdProj ssd_proj(const float* p) const { return SsdProj{p, split, z_at, x_at, dt_at}; }
};

struct Zirurax final : FolderModel {
    Config cfg;
    std::vector<Layer> layers;
    uint32_t pass = 0;  // tokens a prompt pass takes
    // a step's vectors
    float *proj = nullptr, *act = nullptr, *mixed = nullptr, *gated = nullptr, *y_left = nullptr, *y_right = nullptr, *y_mlp = nullptr, *scratch = nullptr;
    // a prompt pass's rows
    float *p_proj = nullptr, *p_gated = nullptr, *p_left = nullptr, *p_right = nullptr, *p_mlp = nullptr, *p_scratch = nullptr, *p_conv = nullptr;
    void *p_act = nullptr, *p_mixed = nullptr, *p_normed = nullptr;
    SsdScratch p_ssd{};

    // a prompt pass's state-space side runs beside its attention
    hipStream_t side = nullptr;
    hipEvent_t projected = nullptr, scanned = nullptr;

    void release(wick_rocm_ctx* ctx) override {
        if (side) (void)hipStreamSynchronize(side), (void)hipStreamDestroy(side);
        if (projected) (void)hipEventDestroy(projected);
        if (scanned) (void)hipEventDestroy(scanned);
        FolderModel::release(ctx);
    }
    bool exact(const Layer& l) const { return f32 || !window_prefill_shape(l.c.left.dim, l.c.left.vdim); }
    int load(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t context_size);
    int load_layer(wick_rocm_ctx* ctx, const wick_safetensors* folder, uint32_t i);
    int enqueue_step(wick_rocm_ctx* ctx, StepMode mode) override;
    int alloc_rows(wick_rocm_ctx* ctx) override;
    int prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                    float* layers_out) override;
    std::vector<StatePiece> state_pieces(uint32_t seq_len) const override;
};

// ---- config.json ------------------------------------------------------------------------------------------------------------

// Frequencies with long wavelengths stretched: fewer than `low` periods within `original` positions by `factor`, more than `high` not
// at all, a ramp in between (Llama 3.1's rule).
std::vector<double> scaled_frequencies(std::vector<double> freqs, const Json& j, const std::string& where) {
    const double factor = number(j, "factor", where), low = number(j, "low", where), high = number(j, "high", where), original = number(j, "original", where);
    if (!(factor > 0.0) || !(original > 0.0) || !(low <= high)) throw ConfigError{"config: " + where + " is out of range"};
    for (double& f : freqs) {
        const double wavelength = 2.0 * M_PI / f;
        if (wavelength < original / high) continue;
        if (wavelength > original / low) {
            f /= factor;
            continue;
        }
        const double s = (original / wavelength - low) / (high - low);
        f = (1.0 - s) * f / factor + s * f;
    }
    return freqs;
}

AttentionConfig attention_config(const Json& j, const std::string& w) {
    AttentionConfig a;
    a.heads = size(j, "heads", w), a.kv_heads = size(j, "kv_heads", w), a.dim = size(j, "dim", w), a.vdim = size(j, "vdim", w);
    a.scale = number(j, "scale", w);
    if (a.heads % a.kv_heads) throw ConfigError{"config: " + w + ": kv_heads must divide heads"};
    if (const Json* m = optional(j, "mask")) a.window = size(*m, "size", w + ".mask");
    if (optional(j, "softcap")) a.softcap = number(j, "softcap", w);
    if (a.softcap < 0.0) throw ConfigError{"config: " + w + ".softcap is out of range"};
    if (const Json* r = optional(j, "rot")) {
        a.rot = size(*r, "dims", w + ".rot");
        const double base = number(*r, "base", w + ".rot");
        if (a.rot % 2u || a.rot > a.dim || !(base > 0.0)) throw ConfigError{"config: " + w + ".rot is out of range"};
        a.freqs = rope_frequencies(base, a.rot);
        if (const Json* s = optional(*r, "scaling")) a.freqs = scaled_frequencies(a.freqs, *s, w + ".rot.scaling");
    }
    return a;
}

SsdConfig ssd_config(const Json& j, const std::string& w) {
    SsdConfig s;
    s.heads = size(j, "heads", w), s.groups = size(j, "groups", w), s.state = size(j, "state", w), s.vdim = size(j, "vdim", w);
    s.conv = size(j, "conv", w), s.parts = size(j, "norm_groups", w);
    if (s.heads % s.groups || (uint64_t)s.heads * s.vdim % s.parts) throw ConfigError{"config: " + w + ": groups must divide heads, norm_groups their width"};
    return s;
}

Config read_config(const Json& j) {
    Config c;
    c.vocab = size(j, "vocab", "config"), c.width = size(j, "width", "config");
    c.eps = number(need(j, "norm", "config"), "eps", "norm");
    c.embed_scale = number(need(j, "embedding", "config"), "scale", "embedding");
    const Json& layers = need(j, "layers", "config");
    if (layers.kind != Json::kArray || layers.items.empty()) throw ConfigError{"config: layers is not a list"};
    for (size_t i = 0; i < layers.items.size(); i++) {
        const std::string w = "layers[" + std::to_string(i) + "]";
        const Json& l = layers.items[i];
        if (text(l, "type", w) != "parallel") throw ConfigError{"config: " + w + ": unknown type " + text(l, "type", w)};
        const Json& m = need(l, "mixer", w);
        LayerConfig lc;
        lc.left = attention_config(need(m, "left", w + ".mixer"), w + ".mixer.left");
        lc.right = ssd_config(need(m, "right", w + ".mixer"), w + ".mixer.right");
        if (const Json* f = optional(l, "mlp")) {
            if (text(*f, "kind", w + ".mlp") != "dense") throw ConfigError{"config: " + w + ".mlp: unknown kind " + text(*f, "kind", w + ".mlp")};
            lc.ff = size(*f, "ff", w + ".mlp");
        }
        c.layers.push_back(lc);
    }
    return c;
}

// ---- weights ----------------------------------------------------------------------------------------------------------------

int Zirurax::load_layer(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t i) {
    const std::string p = "l" + std::to_string(i) + ".", lp = p + "mix.left.", rp = p + "mix.right.", fp = p + "mlp.";
    Layer& l = layers[i];
    l.c = cfg.layers[i];
    const uint32_t D = cfg.width;
    const AttentionConfig& a = l.c.left;
    const SsdConfig& r = l.c.right;
    MODEL_TRY(upload(ctx, widened(tensor(f, p + "norm1", {D}), D), &l.norm));
    MODEL_TRY(upload(ctx, widened(tensor(f, lp + "out", {D}), D), &l.left_gain));
    MODEL_TRY(upload(ctx, widened(tensor(f, rp + "out", {D}), D), &l.right_gain));

    WindowShape& w = l.window;
    w.heads = a.heads, w.kv_heads = a.kv_heads, w.dim = a.dim, w.vdim = a.vdim, w.rot = a.rot;
    window_pads(a.dim, a.vdim, &w.dqp, &w.dvp);
    w.window = a.window, w.max_seq = info.max_seq_len, w.slots = window_slots(a.window, pass, info.max_seq_len);
    w.scale = (float)a.scale, w.softcap = (float)a.softcap, w.f32 = f32;
    MODEL_TRY(upload_rope(ctx, a.freqs, &l.rope));

    SsdShape& s = l.ssd;
    s.heads = r.heads, s.groups = r.groups, s.state = r.state, s.vdim = r.vdim, s.taps = r.conv;
    for (s.np = 32; s.np < r.state;) s.np *= 2;
    s.pp = pad_to(r.vdim, 16);
    const uint32_t inner = l.inner(), H = r.heads, G = r.groups, N = r.state, P = r.vdim, C = s.channels();

    // every projection of the norm in one weight: q | k | v | gate | z | x B C | dt, every head padded with zero rows, and the feed-forward's pairs
    l.q_at = 0, l.k_at = a.heads * w.dqp, l.v_at = l.k_at + a.kv_heads * w.dqp, l.g_at = l.v_at + a.kv_heads * w.dvp, l.z_at = l.g_at + a.heads * w.dvp;
    l.x_at = l.z_at + H * s.pp, l.dt_at = l.x_at + C, l.split = pad_to(l.dt_at + H, kDensePad);
    const uint32_t ffp = pad_to(l.c.ff, kDensePad);
    Packer in(1, l.split + 2 * ffp, D);
    auto heads = [&](uint32_t at, const uint16_t* src, uint32_t count, uint32_t each, uint32_t padded) {
        for (uint32_t h = 0; h < count; h++) in.rows(0, at + h * padded, src + (size_t)h * each * D, each, D);
    };
    heads(l.q_at, tensor(f, lp + "q", {a.heads * a.dim, D}), a.heads, a.dim, w.dqp);
    heads(l.k_at, tensor(f, lp + "k", {a.kv_heads * a.dim, D}), a.kv_heads, a.dim, w.dqp);
    heads(l.v_at, tensor(f, lp + "v", {a.kv_heads * a.vdim, D}), a.kv_heads, a.vdim, w.dvp);
    heads(l.g_at, tensor(f, lp + "g", {a.heads * a.vdim, D}), a.heads, a.vdim, w.dvp);
    const uint16_t* win = tensor(f, rp + "in", {2 * inner + 2 * G * N + H, D});
    auto section = [&](uint32_t row) { return win + (size_t)row * D; };
    heads(l.z_at, section(0), H, P, s.pp);
    heads(l.x_at, section(inner), H, P, s.pp);
    heads(l.x_at + H * s.pp, section(2 * inner), 2 * G, N, s.np);
    heads(l.dt_at, section(2 * inner + 2 * G * N), H, 1, 1);
    if (l.c.ff) {
        const uint16_t *gate = tensor(f, fp + "gate", {l.c.ff, D}), *up = tensor(f, fp + "up", {l.c.ff, D});
        for (uint32_t e = 0; e < l.c.ff; e++) {
            in.row(0, l.split + Packer::paired(e, false), gate + (size_t)e * D, D);
            in.row(0, l.split + Packer::paired(e, true), up + (size_t)e * D, D);
        }
        Packer down(1, D, l.c.ff);
        down.rows(0, 0, tensor(f, fp + "down", {D, l.c.ff}), D, l.c.ff);
        MODEL_TRY(upload(ctx, down, &l.down));
    }
    MODEL_TRY(upload(ctx, in, &l.in));
    Packer left(1, D, a.heads * a.vdim), right(1, D, inner);
    left.rows(0, 0, tensor(f, lp + "o", {D, a.heads * a.vdim}), D, a.heads * a.vdim);
    right.rows(0, 0, tensor(f, rp + "o", {D, inner}), D, inner);
    MODEL_TRY(upload(ctx, left, &l.left_out));
    MODEL_TRY(upload(ctx, right, &l.right_out));

    // the convolution's channels where the projection has them
    auto at = [&](uint32_t ch) {
        if (ch < inner) return ch / P * s.pp + ch % P;
        const uint32_t b = ch - inner;
        return H * s.pp + b / N * s.np + b % N;
    };
    const uint32_t channels = inner + 2 * G * N;
    float *conv = nullptr, *conv_bias = nullptr, *rate = nullptr, *dt_bias = nullptr, *d = nullptr;
    MODEL_TRY(upload(ctx, taps_by_time(tensor(f, rp + "conv", {channels, r.conv}), channels, r.conv, C, at), &conv));
    MODEL_TRY(upload(ctx, taps_by_time(tensor(f, rp + "conv.b", {channels}), channels, 1, C, at), &conv_bias));
    std::vector<float> rates = widened(tensor(f, rp + "A_log", {H}), H);
    for (float& v : rates) v = (float)-std::exp((double)v);
    MODEL_TRY(upload(ctx, rates, &rate));
    MODEL_TRY(upload(ctx, widened(tensor(f, rp + "dt_bias", {H}), H), &dt_bias));
    MODEL_TRY(upload(ctx, widened(tensor(f, rp + "D", {H}), H), &d));
    MODEL_TRY(upload(ctx, widened(tensor(f, rp + "norm", {inner}), inner), &l.ssd_norm));
    l.ssd_w = SsdWeights{conv, conv_bias, rate, dt_bias, d};

    // positions that were never written are read as (weightless) keys and values: whatever the ring holds there has to be finite
    const size_t keys_n = (size_t)w.slots * w.kv_heads * w.dqp, values_n = (size_t)w.slots * w.kv_heads * w.dvp;
    MODEL_TRY(alloc_act(ctx, keys_n, &l.keys));
    MODEL_TRY(alloc_act(ctx, values_n, &l.values));
    const std::vector<char> zeros(std::max(keys_n, values_n) * act_bytes(), 0);
    MODEL_TRY(wick_rocm_upload(ctx, l.keys, zeros.data(), keys_n * act_bytes()));
    MODEL_TRY(wick_rocm_upload(ctx, l.values, zeros.data(), values_n * act_bytes()));
    MODEL_TRY(alloc_t(ctx, (size_t)r.conv * C, &l.ring));
    return alloc_t(ctx, (size_t)H * s.pp * s.np, &l.state);
}

int Zirurax::load(wick_rocm_ctx* ctx, const wick_safetensors* f, uint32_t context_size) {
    cfg = read_config(f->config);
    eps = (float)cfg.eps, embed_scale = (float)cfg.embed_scale;
    strcpy(info.architecture, "Zirurax");
    // what the kernels' on-chip buffers hold
    if (cfg.width > 8192u) throw ConfigError{"width beyond what the kernels take"};
    bool any_exact = f32;
    for (const LayerConfig& l : cfg.layers) {
        const uint64_t inner = (uint64_t)l.right.heads * l.right.vdim;
        if ((uint64_t)l.left.heads * l.left.vdim > 15360u || l.left.dim > 2048u || inner > 15360u || l.right.state > kSsdMaxState || l.right.conv > 8u ||
            l.right.parts > 512u || l.ff > 15360u || l.left.window > 1u << 30)
            throw ConfigError{"a layer's sizes are beyond what the kernels take"};
        if (!window_prefill_shape(l.left.dim, l.left.vdim)) any_exact = true;
    }
    pass = std::min(context_size, any_exact ? kChunkExact : kChunkBf16);
    MODEL_TRY(load_ends(ctx, f, "Zirurax", cfg.vocab, cfg.width, context_size, nullptr));
    float* gain = nullptr;
    MODEL_TRY(upload(ctx, widened(tensor(f, "final.norm", {cfg.width}), cfg.width), &gain));
    final_norm = Gain{1.0f, gain};
    layers.resize(cfg.layers.size());
    for (uint32_t i = 0; i < layers.size(); i++) MODEL_TRY(load_layer(ctx, f, i));
    info.layer_runs = (uint32_t)layers.size();

    uint32_t proj_w = 4, act_w = 4, mixed_w = 4, gated_w = 4;
    size_t scratch_w = 4;
    for (const Layer& l : layers) {
        proj_w = std::max(proj_w, l.split), act_w = std::max(act_w, l.down.kp), mixed_w = std::max(mixed_w, l.left_out.kp), gated_w = std::max(gated_w, l.right_out.kp);
        scratch_w = std::max(scratch_w, window_attention_scratch_floats(l.window, 1));
    }
    MODEL_TRY(alloc_step(ctx));
    MODEL_TRY(alloc_t(ctx, proj_w, &proj));
    MODEL_TRY(alloc_t(ctx, act_w, &act));
    MODEL_TRY(alloc_t(ctx, mixed_w, &mixed));
    MODEL_TRY(alloc_t(ctx, gated_w, &gated));
    MODEL_TRY(alloc_t(ctx, dp, &y_left));
    MODEL_TRY(alloc_t(ctx, dp, &y_right));
    MODEL_TRY(alloc_t(ctx, dp, &y_mlp));
    MODEL_TRY(alloc_t(ctx, scratch_w, &scratch));
    return wick_rocm_sync(ctx);
}

// The three sublayers' outputs that a layer leaves to be added.
RowStage pending_of(const Layer& l, const float* left, const float* right, const float* mlp) {
    RowStage s;
    s.y = left, s.w_post = l.left_gain, s.y2 = right, s.w_post2 = l.right_gain, s.g_post = 0.5f;
    if (l.c.ff) s.add = mlp;
    return s;
}

// ---- one step ----------------------------------------------------------------------------------------------------------------

// Token and position are read on the device; x0 holds the token's embedding row already (set_step, or the previous greedy pick).
// The residual update behind a layer happens in the prologue of the launch that reads the residual next.
int Zirurax::enqueue_step(wick_rocm_ctx* ctx, StepMode mode) {
    const Launch L = ctx->launch();
    const uint32_t D = cfg.width;
    const float* x = x0;
    RowStage pend;
    auto stage = [&](const float* gain, bool keep) {
        GemvIn in;
        in.row = pend;
        in.row.x = x, in.row.x_stride = dp, in.row.y_stride = dp, in.row.g_pre = 1.0f, in.row.w_pre = gain, in.row.eps = eps, in.row.dim = D;
        if (keep && pend.pending()) in.row.x_out = x == xs[0] ? xs[1] : xs[0];
        return in;
    };
    for (const Layer& l : layers) {
        const GemvIn in = stage(l.norm, true);
        MODEL_LAUNCH(launch_gemv_project(l.in, l.split, in, proj, act, L));
        if (in.row.x_out) x = in.row.x_out;
        WindowMerge merge;
        MODEL_LAUNCH(launch_parallel_step(l.window, l.window_proj(proj), l.keys, l.values, scratch, mixed, l.left_out.kp, l.ssd, l.ssd_w, l.ssd_proj(proj), l.ring,
                                          l.state, gated, d_pos, &merge, L));
        GemvSegment left{l.left_out, D, mixed, l.c.left.heads * l.c.left.vdim, y_left};
        if (window_merge_foldable(merge)) left.merge = &merge;
        else if (merge.splits > 1) MODEL_LAUNCH(launch_window_merge(merge, 1, mixed, l.left_out.kp, l.left_out.kp, true, L));
        std::vector<GemvSegment> outs;  // the longest first
        if (l.c.ff) outs.push_back(GemvSegment{l.down, D, act, l.down.kp, y_mlp});
        outs.push_back(left);
        outs.push_back(GemvSegment{l.right_out, D, gated, l.inner(), y_right, l.ssd_norm, l.c.right.parts, eps});
        MODEL_LAUNCH(launch_gemv_segments(outs.data(), (uint32_t)outs.size(), L));
        pend = pending_of(l, y_left, y_right, y_mlp);
    }
    return finish_step(ctx, mode, stage(final_norm.w, false));
}

// ---- prompt passes ------------------------------------------------------------------------------------------------------------

int Zirurax::alloc_rows(wick_rocm_ctx* ctx) {
    uint32_t proj_w = 4, act_w = 8, mixed_w = 8, gated_w = 8, conv_w = 4;
    size_t scratch_n = 4, tiles_n = 8, rows_n = 8, meta_n = 4, sums_n = 4;
    bool any_exact = f32;
    for (const Layer& l : layers) any_exact = any_exact || exact(l);
    const uint32_t few = any_exact ? pass : std::min(pass, kShortMax), chunks = ssd_chunks(pass), rows_conv = f32 ? pass : std::min(pass, kShortMax);
    for (const Layer& l : layers) {
        const SsdShape& s = l.ssd;
        proj_w = std::max(proj_w, l.split), act_w = std::max(act_w, l.down.kp), mixed_w = std::max(mixed_w, l.left_out.kp), gated_w = std::max(gated_w, l.right_out.kp);
        conv_w = std::max(conv_w, s.channels());
        for (uint32_t n = 1; n <= few; n++) scratch_n = std::max(scratch_n, window_attention_scratch_floats(l.window, n));
        if (f32) continue;
        tiles_n = std::max(tiles_n, (size_t)chunks * (s.heads * s.pp + s.groups * s.np) * 64), rows_n = std::max(rows_n, (size_t)chunks * 64 * 2 * s.groups * s.np);
        meta_n = std::max(meta_n, (size_t)chunks * s.heads * (2 * 64 + 1)), sums_n = std::max(sums_n, (size_t)chunks * s.heads * s.pp * s.np);
    }
    const size_t n = pass;
    MODEL_TRY(alloc_pass(ctx, pass));
    MODEL_TRY(alloc_t(ctx, n * proj_w, &p_proj));
    MODEL_TRY(alloc_t(ctx, n * gated_w, &p_gated));
    MODEL_TRY(alloc_t(ctx, n * dp, &p_left));
    MODEL_TRY(alloc_t(ctx, n * dp, &p_right));
    MODEL_TRY(alloc_t(ctx, n * dp, &p_mlp));
    MODEL_TRY(alloc_t(ctx, scratch_n, &p_scratch));
    MODEL_TRY(alloc_t(ctx, (size_t)rows_conv * conv_w, &p_conv));
    MODEL_TRY(alloc_act(ctx, n * act_w, &p_act));
    MODEL_TRY(alloc_act(ctx, n * mixed_w, &p_mixed));
    MODEL_TRY(alloc_act(ctx, n * gated_w, &p_normed));
    if (!f32) {
        MODEL_TRY(alloc_t(ctx, tiles_n, &p_ssd.tiles));
        MODEL_TRY(alloc_t(ctx, rows_n, &p_ssd.rows));
        MODEL_TRY(alloc_t(ctx, meta_n, &p_ssd.meta));
        MODEL_TRY(alloc_t(ctx, sums_n, &p_ssd.sums));
        MODEL_TRY(alloc_t(ctx, 2 * sums_n, &p_ssd.starts));
    }
    MODEL_LAUNCH(hipStreamCreateWithFlags(&side, hipStreamNonBlocking));
    MODEL_LAUNCH(hipEventCreateWithFlags(&projected, hipEventDisableTiming));
    MODEL_LAUNCH(hipEventCreateWithFlags(&scanned, hipEventDisableTiming));
    cap = pass;
    return WICK_ROCM_OK;
}

int Zirurax::prompt_pass(wick_rocm_ctx* ctx, const uint32_t* tokens, uint32_t n, uint32_t pos0, const uint32_t* want, uint32_t n_want, float* logits_out,
                         float* layers_out) {
    const Launch L = ctx->launch();
    const uint32_t D = cfg.width;
    MODEL_TRY(wick_rocm_upload(ctx, p_tokens, tokens, (size_t)n * sizeof(uint32_t)));
    MODEL_LAUNCH(launch_embed_activation(embed, cfg.vocab, D, embed_scale, p_tokens, n, p_x0, dp, nullptr, 0, 0, f32, L));
    const float* x = p_x0;
    RowStage pend;
    for (uint32_t i = 0; i < layers.size(); i++) {
        const Layer& l = layers[i];
        const RowsArgs rows = rows_of(pend, x, Gain{1.0f, l.norm}, true, n, pos0);
        MODEL_LAUNCH(launch_rows(rows, kRowNorm, L));
        if (rows.s.x_out) x = rows.s.x_out;
        MODEL_LAUNCH(launch_gemm_project(l.in, GemmIn{p_h, dp, n, f32}, l.split, p_proj, l.split, p_act, l.down.kp, L));
        const WindowProj w = l.window_proj(p_proj);
        const uint32_t lda = l.left_out.kp, ldg = l.right_out.kp;
        const bool fork = n > kForkMin && !(L.timer && L.timer->enabled);
        Launch S = L;
        if (fork) {
            S.stream = side;
            MODEL_LAUNCH(hipEventRecord(projected, L.stream));
            MODEL_LAUNCH(hipStreamWaitEvent(side, projected, 0));
        }
        if (f32 || n <= kShortMax)
            MODEL_LAUNCH(launch_ssd_scan(l.ssd, l.ssd_w, l.ssd_proj(p_proj), l.ring, l.state, p_conv, n, pos0, p_gated, ldg, S));
        else
            MODEL_LAUNCH(launch_ssd_chunks(l.ssd, l.ssd_w, l.ssd_proj(p_proj), l.ring, l.state, p_ssd, n, pos0, p_gated, ldg, S));
        MODEL_LAUNCH(launch_part_norm(p_gated, ldg, n, l.inner(), l.c.right.parts, l.ssd_norm, eps, p_normed, ldg, ldg, f32, S));
        if (fork) MODEL_LAUNCH(hipEventRecord(scanned, side));
        MODEL_LAUNCH(launch_window_store(l.window, w, l.keys, l.values, n, pos0, L));
        if (exact(l) || n <= kShortMax)
            MODEL_LAUNCH(launch_window_attention(l.window, w, l.keys, l.values, p_scratch, n, pos0, nullptr, p_mixed, lda, lda, f32, L));
        else
            MODEL_LAUNCH(launch_window_prefill(l.window, w, l.keys, l.values, n, pos0, static_cast<uint16_t*>(p_mixed), lda, lda, L));
        if (fork) MODEL_LAUNCH(hipStreamWaitEvent(L.stream, scanned, 0));
        const GemmStore outs[3] = {{l.left_out, GemmIn{p_mixed, lda, n, f32}, p_left, dp},
                                   {l.right_out, GemmIn{p_normed, ldg, n, f32}, p_right, dp},
                                   {l.down, GemmIn{p_act, l.down.kp, n, f32}, p_mlp, dp}};
        MODEL_LAUNCH(launch_gemm_stores(outs, l.c.ff ? 3 : 2, L));
        pend = pending_of(l, p_left, p_right, p_mlp);
        if (layers_out) MODEL_TRY(copy_residual(ctx, pend, x, n, layers_out + (size_t)i * n * D));
    }
    return wanted_logits(ctx, pend, x, want, n_want, logits_out);
}

// ---- state --------------------------------------------------------------------------------------------------------------------

std::vector<StatePiece> Zirurax::state_pieces(uint32_t seq_len) const {
    std::vector<StatePiece> v;
    for (const Layer& l : layers) {
        const WindowShape& w = l.window;
        const size_t rows = std::min(seq_len, w.slots);
        if (rows) {
            v.push_back({l.keys, rows * w.kv_heads * w.dqp * act_bytes()});
            v.push_back({l.values, pad_to((uint32_t)rows, 64) * (size_t)w.kv_heads * w.dvp * act_bytes()});
        }
        v.push_back({l.ring, (size_t)l.c.right.conv * l.ssd.channels() * sizeof(float)});
        v.push_back({l.state, (size_t)l.ssd.heads * l.ssd.pp * l.ssd.np * sizeof(float)});
    }
    return v;
}

}  // namespace

int load_zirurax(wick_rocm_ctx* ctx, const wick_safetensors* folder, int dtype, uint32_t context_size, wick_rocm_model** out) {
    return load_folder_model<Zirurax>(ctx, folder, dtype, context_size, out);
}
