// Internal declarations of the bf16 / f32 model path: weights in bfloat16, activations in bfloat16 (matrix products on the matrix
// cores, f32 accumulation) or in f32 (true f32 products), everything else f32.  Not installed.
//
// Layout rules shared by all kernels here:
//   - a weight is row-major [m][kp] bfloat16 with k padded to kp (a multiple of 64, zeros) and m padded to mp (a multiple of 64,
//     zero rows), so that no product needs an edge case in K and a padded output feature comes out as 0;
//   - an activation row has kp elements of the consumer's K, the padding written as zeros by whoever writes the row;
//   - two weights whose outputs are combined element by element (gate / up, the two gates of a recurrence) are interleaved in
//     groups of 16 rows: rows 32 j .. 32 j + 15 are the first weight's features 16 j .., rows 32 j + 16 .. the second's.
#pragma once

#include "wick_rocm_internal.h"

namespace wick_rocm {

constexpr uint32_t pad_to(uint32_t v, uint32_t a) { return (v + a - 1) / a * a; }
constexpr uint32_t kDensePad = 64;

struct DenseWeight {
    uint16_t* d = nullptr;
    uint32_t mp = 0, kp = 0;   // padded rows / columns of one group
    size_t stride = 0;         // elements between groups (experts, blocks); 0: one group
};

// ---- grouped-query attention over a window (windowed_attention.hip) ---------------------------------------------------------------
// Position i sees j with i - window < j <= i (window 0: every j <= i); query head h uses key / value head h / (heads / kv_heads);
// scores are capped, the weighted values gated: out = sigmoid(gate) * sum.  The cache is a ring of `slots` positions, a multiple of 64
// that holds a window and a portion: keys [slots][kv_heads][dqp], values in tiles of 64 positions [slots / 64][kv_heads][dvp][64],
// zeros behind dim / vdim; bfloat16, or f32.
constexpr uint32_t kWindowTile = 64;
struct WindowShape {
    uint32_t heads, kv_heads, dim, vdim;
    uint32_t dqp, dvp;           // multiples of 32
    uint32_t rot;                // coordinates of a head that turn, in pairs (2i, 2i + 1); even
    uint32_t window, slots, max_seq;
    float scale, softcap;        // softcap 0: none
    bool f32;                    // element type of the cache
    __host__ __device__ uint32_t first_seen(uint32_t pos) const { return window && pos + 1u > window ? pos + 1u - window : 0u; }
    // Tiles of the window of `pos`: the first one and how many.
    __host__ __device__ uint32_t window_tiles(uint32_t pos, uint32_t& tile0) const {
        tile0 = first_seen(pos) / kWindowTile;
        return pos / kWindowTile - tile0 + 1u;
    }
};
// Columns of a projection [n][ldp]: q [heads][dqp], k [kv_heads][dqp], v [kv_heads][dvp], g [heads][dvp]; multiples of 4.
struct WindowProj {
    const float* p;
    uint32_t ldp, q_at, k_at, v_at, g_at;
    const float* rope;           // [max_seq][rot / 2][2]: cosine, sine
};
// Partial results of `splits` workgroups along the window, [n][heads][splits][dvp + 4]: {max, sum, -, -, weighted values}.
struct WindowMerge {
    WindowShape s;
    WindowProj w;
    const float* part;
    uint32_t pos0, splits;
    const uint32_t* d_pos;       // non-null: one token at *d_pos
};

// ---- the residual stream between two sublayers (row_ops.hip, and the prologues of dense_gemv.hip) --------------------------
// x_out = x + g_post * y / rms(y) (y null: x_out = x), then h = g_pre * x_out / rms(x_out), optionally with a causal convolution
// over time added: h_t + sum_j conv[j] * h_(t - taps + 1 + j).  The inputs h of the last `taps` positions live in a ring of `taps`
// rows: position p in slot p % taps, so a step overwrites only what no later position needs.
struct RowStage {
    const float* x = nullptr;      // [n][x_stride]
    uint32_t x_stride = 0;
    const float* y = nullptr;      // [n][y_stride]; null: no update
    uint32_t y_stride = 0;
    float g_post = 0.0f, g_pre = 0.0f, eps = 0.0f;
    uint32_t dim = 0;
    float* x_out = nullptr;        // [n][x_stride], never aliases x; null: not kept
    const float* conv = nullptr;   // [taps][x_stride]; null: no convolution
    float* ring = nullptr;         // [taps][x_stride]
    uint32_t taps = 0;
    // y as the weighted outputs of routed experts: y += (1 / top) * sum_s experts[slot(t, s)] (prompt passes only)
    const float* experts = nullptr;     // [n * top][y_stride]
    const uint32_t* slots = nullptr;    // [n][top]: the entry that holds expert s of token t
    uint32_t top = 0;
    // gains per coordinate, and the outputs of sublayers that read the same norm: x_out = x + g_post * (w_post * y / rms(y)
    // + w_post2 * y2 / rms(y2)) + add, h = g_pre * w_pre * x_out / rms(x_out)
    const float *w_pre = nullptr, *w_post = nullptr;    // [dim]; null: ones
    const float *y2 = nullptr, *w_post2 = nullptr;      // [n][y_stride], [dim]; y2 needs y
    const float* add = nullptr;                         // [n][y_stride]
    __host__ __device__ bool pending() const { return y || experts || add; }
    __host__ __device__ bool vector_gains() const { return w_pre || w_post || y2 || add; }
};

// ---- matrix products of a prompt (dense_gemm.hip) ---------------------------------------------------------------------------
// All take activations x [n][ldx] (bfloat16, or f32 with f32 = true).
struct GemmIn {
    const void* x;
    uint32_t ldx, n;
    bool f32;
};
// Rows of x that go through the group's own weight: tile i covers entries first .. first + count - 1 of group `group`.
struct GroupTile {
    uint32_t group, first, count;
};
struct Grouping {
    const GroupTile* tiles = nullptr;    // null: not grouped
    const uint32_t* n_tiles = nullptr;   // on the device
    uint32_t max_tiles = 0;
    const uint32_t* gather = nullptr;    // entry -> row of x; null: entry i is row i
};
constexpr uint32_t kGroupTileRows = 64;
// out[t][f] = W x (+ add[f]), f32.
hipError_t launch_gemm_store(const DenseWeight& w, const GemmIn& in, float* out, uint32_t ldo, const float* add, const Launch& L,
                             const Grouping& g = Grouping());
// Several of the plain ones in one launch (bfloat16; the f32 model's go one by one).
struct GemmStore {
    DenseWeight w;
    GemmIn in;
    float* out;
    uint32_t ldo;
};
constexpr uint32_t kMaxStores = 4;
hipError_t launch_gemm_stores(const GemmStore* g, uint32_t count, const Launch& L);
// out[t][f] = f < split ? gelu_tanh(W x + bias) : W x + bias, f32.
hipError_t launch_gemm_gelu_split(const DenseWeight& w, const GemmIn& in, float* out, uint32_t ldo, const float* bias, uint32_t split, const Launch& L);
// out[t][f] = relu(W x)^2 in the activation type.
hipError_t launch_gemm_relu2(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, const Launch& L);
// out[t][f] = silu(gate) * up (* row_scale[t]) of an interleaved weight, in the activation type.
hipError_t launch_gemm_silu(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, const float* row_scale, const Launch& L,
                            const Grouping& g = Grouping());
// Several projections of one input in one product: rows below `split` (a multiple of 64) are stored as f32, out[t][f]; the interleaved
// pairs behind them become act[t][j] = gelu_tanh(gate) * up in the activation type.
hipError_t launch_gemm_project(const DenseWeight& w, const GemmIn& in, uint32_t split, float* out, uint32_t ldo, void* act, uint32_t lda, const Launch& L);
// out[t][f] = W x in the activation type, or transposed: out[f][t] (ldo >= n rounded up to 4).
hipError_t launch_gemm_convert(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, bool transposed, const Launch& L);
// The gates of a real-gated linear recurrence, block-diagonal: per block b an interleaved weight over the block's columns of x;
// r = sigmoid(.. + r_bias), i = sigmoid(.. + i_bias), log a = r * rate, a = exp(log a), b = sqrt(1 - a^2) * i * u.
struct GateArgs {
    const float *r_bias, *i_bias, *rate, *u;   // [channels]; u: [n][channels]
    float *a, *b;                              // [n][channels]
    uint32_t channels;
};
hipError_t launch_gemm_gates(const DenseWeight& w, const GemmIn& in, uint32_t blocks, uint32_t x_block_stride, const GateArgs& g, const Launch& L);

// ---- matrix-vector products of one token (dense_gemv.hip): f32 activations, bfloat16 weights --------------------------------
enum GemvAct { kActNone = 0, kActGeluSplit = 1, kActRelu2 = 2 };
// out = act(W v + bias); v = vec (in.vec non-null), or the row stage's h, or [x_out | x0] of the row stage (loop entry).
struct GemvIn {
    const float* vec = nullptr;
    RowStage row;
    const float* x0 = nullptr;
    uint32_t x0_at = 0;             // the column of x0 in the weight's K
    uint32_t k = 0;                 // columns of the weight that are used (a multiple of 8); 0: all of them
    uint32_t vec_len = 0;           // floats of vec (zeros are taken behind them); 0: k
    const uint32_t* d_pos = nullptr;
};
hipError_t launch_gemv_dense(const DenseWeight& w, uint32_t m, const GemvIn& in, float* out, const float* bias, int act, uint32_t split, const Launch& L);
// The step's counterpart of launch_gemm_project: out[f] below `split`, act[j] behind it.
hipError_t launch_gemv_project(const DenseWeight& w, uint32_t split, const GemvIn& in, float* out, float* act, const Launch& L);
// Up to kMaxSegments products of their own vectors in one launch; with norm_w the vector is first normed in `parts` equal parts.
struct GemvSegment {
    DenseWeight w;
    uint32_t m;
    const float* vec;
    uint32_t vec_len;              // floats of vec (zeros are taken behind them)
    float* out;
    const float* norm_w = nullptr; // [vec_len]
    uint32_t parts = 1;
    float eps = 0.0f;
    const WindowMerge* merge = nullptr;  // at most one segment: the vector is what these partials of an attention step come to (vec is not read)
};
constexpr uint32_t kMaxSegments = 4;
hipError_t launch_gemv_segments(const GemvSegment* segs, uint32_t count, const Launch& L);
// Routed gated feed-forward of one token: act_e[s][ffp] = silu(gate) * up of expert table[token][s], act_s[..] of the shared one,
// shared_gate[0] = sigmoid(w_sg . h).
struct RoutedMlp {
    DenseWeight gate_up, down;               // experts: [experts] groups
    DenseWeight shared_gate_up, shared_down; // shared_gate_up.d null: none
    const uint16_t* shared_sg = nullptr;     // [kp]
    const int32_t* table = nullptr;          // [vocab][top]
    uint32_t top = 0, experts = 0;
};
hipError_t launch_gemv_routed_up(const RoutedMlp& m, const GemvIn& in, const uint32_t* d_token, float* act, const Launch& L);
// out[f] = (1 / top) * sum_s W_down,e(s) act_e[s] + shared_gate * W_down,shared act_s.
hipError_t launch_gemv_routed_down(const RoutedMlp& m, uint32_t rows, const float* act, const uint32_t* d_token, float* out, const Launch& L);
// Floats of the act buffer the two share: [top][ffp] | [shared ffp] | gate.
uint32_t routed_act_floats(const RoutedMlp& m);

// ---- rows of a prompt (row_ops.hip) -------------------------------------------------------------------------------------------
enum RowOut {
    kRowNorm = 0,   // h -> out
    kRowSplit = 1,  // x_out itself -> out as two terms (bfloat16: hi in columns [0, kp), lo in [lo_at, lo_at + kp)); f32: one term
    kRowOnly = 2    // x_out only
};
struct RowsArgs {
    RowStage s;
    uint32_t n = 0, pos0 = 0;
    const uint32_t* rows = nullptr;   // row r of the output is token rows[r]; null: r (no convolution with rows)
    void* out = nullptr;
    uint32_t ldo = 0, kp = 0;         // output row stride, padded columns to write
    uint32_t lo_at = 0;
    bool f32 = false;
    const uint16_t* gate_w = nullptr; // [kp]: row_gate[r] = sigmoid(gate_w . h)
    float* row_gate = nullptr;
};
hipError_t launch_rows(const RowsArgs& a, int mode, const Launch& L);
uint32_t rows_max_dim(uint32_t taps);
// out[t] = w * y[t] / rms in `parts` equal parts of the row, in the activation type (kp columns, zeros behind dim).
hipError_t launch_part_norm(const float* y, uint32_t ldy, uint32_t n, uint32_t dim, uint32_t parts, const float* w, float eps, void* out, uint32_t ldo, uint32_t kp,
                            bool f32, const Launch& L);
// Embedding rows * scale -> x f32 [n][x_stride] and, when given, the activation form at xa [n][ldo] (kp columns).
hipError_t launch_embed_activation(const uint16_t* embed, uint32_t vocab, uint32_t dim, float scale, const uint32_t* tokens, uint32_t n, float* x, uint32_t x_stride, void* xa,
                                   uint32_t ldo, uint32_t kp, bool f32, const Launch& L);
// Groups the n * top (token, expert) pairs of one table by expert: entry_token[e], slot_of[t][s], tiles of kGroupTileRows entries.
struct RouteJob {
    const int32_t* table;
    uint32_t top, experts;
    uint32_t *entry_token, *slot_of, *n_tiles;
    GroupTile* tiles;
};
constexpr uint32_t kRouteMaxExperts = 4096;
hipError_t launch_route(const RouteJob* d_jobs, uint32_t n_jobs, const uint32_t* tokens, uint32_t n, const Launch& L);
inline uint32_t route_max_tiles(uint32_t n, uint32_t top, uint32_t experts) {
    const uint32_t entries = n * top;
    return entries / kGroupTileRows + (experts < entries ? experts : entries);
}

// ---- the recurrent block (rglru.hip) --------------------------------------------------------------------------------------------
// u = conv(x) + conv_bias over [n] tokens; x are columns [x_at, x_at + channels) of proj [n][ldp].  The ring holds the last `taps`
// inputs like RowStage's.  u32: [n][channels] f32; ua: activation form, per block of bp channels hi | lo (bfloat16) or one term (f32).
struct RecurrentConv {
    const float* proj;
    uint32_t ldp, x_at, channels, block, taps, pos0;
    const float *w, *bias;   // [taps][channels], [channels]
    float* ring;
    float* u;
    void* ua;
    uint32_t lda;
    bool f32;
};
hipError_t launch_recurrent_conv(const RecurrentConv& a, uint32_t n, const Launch& L);
// S_t = a_t S_(t-1) + b_t; out[t] = S_t * y_t (activation form, kp columns, zeros behind the channels).  The state is read when
// pos0 > 0 and written.  scratch: recurrent_scan_scratch_floats.
size_t recurrent_scan_scratch_floats(uint32_t n, uint32_t channels);
hipError_t launch_recurrent_scan(const float* a, const float* b, const float* y, uint32_t ldy, float* state, uint32_t n, uint32_t channels, uint32_t pos0,
                                 void* out, uint32_t ldo, uint32_t kp, bool f32, float* scratch, const Launch& L);
// One token: convolution, gates, state update and S * y in one launch.  gates: [blocks] interleaved groups over the block's columns
// (kp = terms * block; only the first `block` columns are used here).
struct RecurrentStep {
    const float* proj;       // [y (channels, after its activation) | x (channels)]
    uint32_t channels, block, blocks, taps;
    const float *conv_w, *conv_bias;
    float *ring, *state;
    DenseWeight gates;
    const float *r_bias, *i_bias, *rate;
    float* out;              // [channels]
    const uint32_t* d_pos;
};
hipError_t launch_recurrent_step(const RecurrentStep& a, const Launch& L);

// ---- attention over a cached latent (latent_attention.hip) ------------------------------------------------------------------------
// A cache row is [latent (rank, padded to rank_p) | rotated key part (rot, padded to rot_p)], zeros in the padding; bfloat16, or f32.
struct LatentShape {
    uint32_t heads, dim, rot, vdim, rank;
    uint32_t rank_p, rot_p;      // multiples of 32, a multiple of 64 together
    __host__ __device__ uint32_t row() const { return rank_p + rot_p; }
    float scale, eps;
    uint32_t max_seq;
    bool f32;                    // element type of the cache
};
struct LatentWeights {
    const uint16_t *uk, *uv;     // [heads * dim][rank_p], [heads * vdim][rank_p]
    const float* norm;           // [rank]
    const float* rope;           // [max_seq][rot / 2][2]: cosine, sine
};
// proj: [n][ldp] = [q (heads * (dim + rot)) | latent | rotated key part]; rows of the cache for positions pos0 ..
// and the absorbed queries qa [n][heads][row()] = [W_uk^T q | rotated q part].
hipError_t launch_latent_absorb(const LatentShape& s, const LatentWeights& w, const float* proj, uint32_t ldp, void* cache, float* qa, uint32_t n,
                                uint32_t pos0, const uint32_t* d_pos, const Launch& L);
// The same without absorbing: the rotated queries as bfloat16 terms hi | lo, [n][heads][2][dqp].
hipError_t launch_latent_rope(const LatentShape& s, const LatentWeights& w, const float* proj, uint32_t ldp, void* cache, uint16_t* q, uint32_t dqp,
                              uint32_t n, uint32_t pos0, const Launch& L);
// Causal attention of absorbed queries over the cache, split over the sequence, and the value expansion:
// out[t][h * vdim ..] f32, or the activation form with kp columns.
size_t latent_attention_scratch_floats(const LatentShape& s, uint32_t n);
uint32_t latent_attention_splits(const LatentShape& s, uint32_t n);
hipError_t launch_latent_attention(const LatentShape& s, const LatentWeights& w, const float* qa, const void* cache, float* scratch, uint32_t n,
                                   uint32_t pos0, const uint32_t* d_pos, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L);
// Causal attention of a prompt over expanded keys kx [keys][ldk] (a row: [heads][dqp]) and values vt [heads * dvp][ldv] (both bfloat16).
bool latent_prefill_shape(uint32_t dim, uint32_t rot, uint32_t vdim, uint32_t* dqp, uint32_t* dvp);
hipError_t launch_latent_prefill(const LatentShape& s, const uint16_t* q, const uint16_t* kx, uint32_t ldk, const uint16_t* vt, uint32_t ldv, uint32_t dqp,
                                 uint32_t dvp, uint32_t n, uint32_t pos0, uint16_t* out, uint32_t ldo, uint32_t kp, const Launch& L);

// Launches of windowed attention (windowed_attention.hip).
uint32_t window_slots(uint32_t window, uint32_t portion, uint32_t max_seq);
bool window_prefill_shape(uint32_t dim, uint32_t vdim);   // dqp / dvp of the next function have matrix-core kernels
void window_pads(uint32_t dim, uint32_t vdim, uint32_t* dqp, uint32_t* dvp);
size_t window_attention_scratch_floats(const WindowShape& s, uint32_t n);
// Keys (rotated) and values of n tokens into the cache.
hipError_t launch_window_store(const WindowShape& s, const WindowProj& w, void* kc, void* vc, uint32_t n, uint32_t pos0, const Launch& L);
// n tokens over the cache, all arithmetic f32: out[t][h * vdim ..] f32 or the activation form (kp columns).  With d_pos: one token at
// *d_pos whose key and value are not in the cache yet; they are appended.
hipError_t launch_window_attention(const WindowShape& s, const WindowProj& w, void* kc, void* vc, float* scratch, uint32_t n, uint32_t pos0,
                                   const uint32_t* d_pos, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L);
// Partials to out[t][h * vdim ..], gated.  Foldable ones (a step's) can go into the product that reads them, GemvSegment::merge.
hipError_t launch_window_merge(const WindowMerge& m, uint32_t n, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L);
bool window_merge_foldable(const WindowMerge& m);
// A prompt's queries on the matrix cores (bfloat16 cache, window_prefill_shape).
hipError_t launch_window_prefill(const WindowShape& s, const WindowProj& w, const void* kc, const void* vc, uint32_t n, uint32_t pos0, uint16_t* out,
                                 uint32_t ldo, uint32_t kp, const Launch& L);

// ---- state-space duality (ssd.hip) --------------------------------------------------------------------------------------------------
// Per head a state S [vdim][state]: S_t = exp(rate dt_t) S_(t-1) + dt_t x_t B_t^T, y_t = S_t C_t + D x_t, out = y * silu(z); x, B, C
// behind a short convolution with silu, dt = softplus(. + dt_bias).  Channels of the convolution: [x: heads * pp | B: groups * np |
// C: groups * np], vdim and state padded with zero channels.
struct SsdShape {
    uint32_t heads, groups, state, vdim, taps;
    uint32_t np, pp;             // state to a power of two >= 32, vdim to a multiple of 16
    __host__ __device__ uint32_t channels() const { return heads * pp + 2u * groups * np; }
};
struct SsdWeights {
    const float *conv, *conv_bias;          // [taps][channels], [channels]
    const float *rate, *dt_bias, *d;        // [heads]; rate = -exp(A_log)
};
// Columns of a projection [n][ldp]: z [heads][pp], the convolution's channels at x_at, dt [heads].
struct SsdProj {
    const float* p;
    uint32_t ldp, z_at, x_at, dt_at;
};
constexpr uint32_t kSsdMaxState = 512;
// One token: convolution, state and gate; out [heads * vdim] f32.
hipError_t launch_ssd_step(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, float* out, const uint32_t* d_pos, const Launch& L);
// The same beside a step of windowed attention over the same projection, in one launch (parallel_step.hip): `merge` describes the
// attention's partials that are left in scratch; with one split its result is in `attended` already and merge.splits is 1.
hipError_t launch_parallel_step(const WindowShape& s, const WindowProj& w, void* kc, void* vc, float* scratch, float* attended, uint32_t attended_len,
                                const SsdShape& ss, const SsdWeights& sw, const SsdProj& sp, float* ring, float* state, float* out, const uint32_t* d_pos,
                                WindowMerge* merge, const Launch& L);
// A portion, token by token in f32 (rows: [n][channels] scratch).  out [n][ldo] f32.
hipError_t launch_ssd_scan(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, float* rows, uint32_t n, uint32_t pos0,
                           float* out, uint32_t ldo, const Launch& L);
// A portion in chunks of 64 tokens on the matrix cores.
struct SsdScratch {
    uint16_t *tiles, *rows;      // [chunks][heads * pp + groups * np][64], [chunks * 64][2 * groups * np]
    float* meta;                 // [chunks][heads][2][64] | [chunks][heads]
    float* sums;                 // [chunks][heads * pp * np]: a chunk's own contribution to the state
    uint16_t* starts;            // [chunks][heads][2][pp * np]: the state in front of a chunk, hi | lo
};
inline uint32_t ssd_chunks(uint32_t n) { return (n + 63u) / 64u; }
hipError_t launch_ssd_chunks(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, const SsdScratch& scratch, uint32_t n,
                             uint32_t pos0, float* out, uint32_t ldo, const Launch& L);

}  // namespace wick_rocm
