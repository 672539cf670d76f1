// Rows of a prompt between the matrix products: the residual update with its norms, the input convolution, embedding rows and the
// grouping of tokens by expert.  Everything is computed in f32; rows leave in the activation type of the next product.
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));

constexpr uint32_t kRowsLdsBytes = 160u * 1024u;

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(uint16_t* p, float v) { *p = __builtin_bit_cast(uint16_t, (__bf16)v); }

__device__ __forceinline__ void store4(float* p, v4f v) { *reinterpret_cast<v4f*>(p) = v; }
__device__ __forceinline__ void store4(uint16_t* p, v4f v) {
    bf4 b;
#pragma unroll
    for (int i = 0; i < 4; i++) b[i] = (__bf16)v[i];
    *reinterpret_cast<bf4*>(p) = b;
}

// y of token t at coordinate e: the sublayer's output, or the mean of the routed experts' outputs on top of it.
__device__ __forceinline__ float row_y(const RowStage& s, uint32_t t, uint32_t e) {
    float v = s.y ? s.y[(size_t)t * s.y_stride + e] : 0.0f;
    if (s.experts) {
        float m = 0.0f;
        for (uint32_t k = 0; k < s.top; k++) m += s.experts[(size_t)s.slots[(size_t)t * s.top + k] * s.y_stride + e];
        v += m / (float)s.top;
    }
    return v;
}

// One row by the calling wave: dst[0 .. dim) = the updated residual, normed when NORM.  dst may be LDS or global memory; a lane
// only re-reads what it wrote itself.
template <bool NORM>
__device__ __forceinline__ void stage_row(const RowStage& s, uint32_t t, float* dst, float* x_out) {
    const uint32_t lane = threadIdx.x & 63u;
    const float* x = s.x + (size_t)t * s.x_stride;
    const float *y2 = s.y2 ? s.y2 + (size_t)t * s.y_stride : nullptr, *add = s.add ? s.add + (size_t)t * s.y_stride : nullptr;
    const bool has_y = s.y || s.experts;
    float sy = 0.0f, sy2 = 0.0f;
    if (has_y) {
        float ss = 0.0f, ss2 = 0.0f;
        for (uint32_t e = lane; e < s.dim; e += 64) {
            const float v = row_y(s, t, e);
            ss += v * v;
            if (y2) ss2 += y2[e] * y2[e];
        }
        sy = s.g_post / sqrtf(wave_sum_f32(ss) / (float)s.dim + s.eps);
        if (y2) sy2 = s.g_post / sqrtf(wave_sum_f32(ss2) / (float)s.dim + s.eps);
    }
    float ss = 0.0f;
    for (uint32_t e = lane; e < s.dim; e += 64) {
        float v = x[e];
        if (has_y) v += row_y(s, t, e) * sy * (s.w_post ? s.w_post[e] : 1.0f);
        if (y2) v += y2[e] * sy2 * (s.w_post2 ? s.w_post2[e] : 1.0f);
        if (add) v += add[e];
        dst[e] = v;
        if (x_out) x_out[e] = v;
        ss += v * v;
    }
    if constexpr (NORM) {
        const float sx = s.g_pre / sqrtf(wave_sum_f32(ss) / (float)s.dim + s.eps);
        for (uint32_t e = lane; e < s.dim; e += 64) dst[e] *= s.w_pre ? sx * s.w_pre[e] : sx;
    }
}

// The general form (any width and number of taps the LDS holds).  A workgroup takes `tile` consecutive rows; with a convolution it also stages the taps - 1 rows in front of them (from its own
// inputs, or from the ring for positions before this portion).  Only the first workgroup reads the ring (tile >= taps - 1), and it
// alone writes it, after its reads: the last rows of the portion, recomputed.
template <int MODE, bool CONV, typename AT>
__global__ __launch_bounds__(256) void rows_kernel(RowsArgs a, uint32_t tile) {
    extern __shared__ float hrow[];
    const RowStage& s = a.s;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, j0 = blockIdx.x * tile, dim = s.dim;
    const uint32_t halo = CONV ? s.taps - 1u : 0u;
    for (uint32_t r = wave; r < tile + halo; r += 4) {
        const int j = (int)j0 - (int)halo + (int)r;
        if (j >= (int)a.n) break;
        float* h = hrow + (size_t)r * dim;
        if (j < 0) {
            const int p = (int)a.pos0 + j;
            const float* past = p >= 0 ? s.ring + (size_t)((uint32_t)p % s.taps) * s.x_stride : nullptr;
            for (uint32_t e = lane; e < dim; e += 64) h[e] = past ? past[e] : 0.0f;
            continue;
        }
        const uint32_t t = a.rows ? a.rows[j] : (uint32_t)j;
        stage_row<MODE == kRowNorm>(s, t, h, s.x_out && r >= halo ? s.x_out + (size_t)t * s.x_stride : nullptr);
        if (MODE == kRowNorm && a.gate_w && r >= halo) {
            float d = 0.0f;
            for (uint32_t e = lane; e < dim; e += 64) d += h[e] * __uint_as_float((uint32_t)a.gate_w[e] << 16);
            d = wave_sum_f32(d);
            if (lane == 0) a.row_gate[j] = 1.0f / (1.0f + expf(-d));
        }
    }
    if (MODE == kRowOnly) return;
    __syncthreads();
    const uint32_t rows = a.n - j0 < tile ? a.n - j0 : tile;
    AT* out = static_cast<AT*>(a.out) + (size_t)j0 * a.ldo;
    for (uint32_t e = tid; e < a.kp; e += 256) {
        for (uint32_t r = 0; r < rows; r++) {
            float v = 0.0f;
            if (e < dim) {
                v = hrow[(size_t)(r + halo) * dim + e];
                if constexpr (CONV) {
                    const float h = v;
                    float c = 0.0f;
                    for (uint32_t k = 0; k < s.taps; k++) c += s.conv[(size_t)k * s.x_stride + e] * hrow[(size_t)(r + k) * dim + e];
                    v = h + c;
                }
            }
            AT* o = out + (size_t)r * a.ldo + e;
            if (MODE == kRowSplit && sizeof(AT) == 2) {
                const float hi = (float)(__bf16)v;
                put(o, hi), put(o + a.lo_at, v - hi);
            } else {
                put(o, v);
            }
        }
    }
    if (CONV && blockIdx.x == 0) {
        const uint32_t first = a.n > s.taps ? a.n - s.taps : 0u;
        for (uint32_t j = first + wave; j < a.n; j += 4) stage_row<true>(s, j, s.ring + (size_t)((a.pos0 + j) % s.taps) * s.x_stride, nullptr);
    }
}

// ---- the fast form: up to four taps, up to 4096 coordinates -------------------------------------------------------------------
// A thread owns four neighbouring coordinates of R consecutive rows and keeps them in registers: all loads of the tile are in flight
// together, the R sums of squares go through one exchange, and the convolution, which runs along the rows, never leaves the thread.
constexpr int kHalo = 3;

__device__ __forceinline__ v4f load4(const float* p) { return *reinterpret_cast<const v4f*>(p); }
__device__ __forceinline__ v4f mask4(v4f v, uint32_t e, uint32_t dim) {
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (e + i >= dim) v[i] = 0.0f;
    return v;
}
__device__ __forceinline__ v4f load_gain(const float* w, uint32_t e, uint32_t dim) {  // (a gain's row ends at dim)
    v4f v;
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = e + i < dim ? w[e + i] : 0.0f;
    return v;
}
__device__ __forceinline__ float dot4(v4f a, v4f b) { return (a[0] * b[0] + a[1] * b[1]) + (a[2] * b[2] + a[3] * b[3]); }

// sum[r] over the workgroup for R values per thread.  red: [R][NT / 64].
template <int R, int NT>
__device__ __forceinline__ void block_sums(float (&v)[R], float* red) {
    constexpr int W = NT / 64;
    __syncthreads();  // red may still be read from an earlier call
#pragma unroll
    for (int r = 0; r < R; r++) {
        const float w = wave_sum_f32(v[r]);
        if ((threadIdx.x & 63u) == 0) red[r * W + (threadIdx.x >> 6)] = w;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < R; r++) {
        float t = 0.0f;
#pragma unroll
        for (int w = 0; w < W; w++) t += red[r * W + w];
        v[r] = t;
    }
}

// Rows first .. first + R - 1 (clamped to n - 1; negative ones are left at zero): h[r] = the updated residual, normed when NORM;
// rows from `own` on are stored to x_out.  GAINS: gains per coordinate, the second normed and the plain addend.
template <bool NORM, bool GAINS, int R, int NT>
__device__ __forceinline__ void stage_tile(const RowsArgs& a, int first, int own, v4f (&h)[R], float* red) {
    const RowStage& s = a.s;
    const uint32_t e = 4u * threadIdx.x;
    const bool on = e < s.dim, has_y = s.y || s.experts;
    v4f y[R], y2[GAINS ? R : 1], add[GAINS ? R : 1];
    v4f wp, wp2, wn;
    uint32_t row[R];
    if constexpr (GAINS) {
        const v4f one = {1.f, 1.f, 1.f, 1.f};
        wp = on && s.w_post ? load_gain(s.w_post, e, s.dim) : one, wp2 = on && s.w_post2 ? load_gain(s.w_post2, e, s.dim) : one;
        wn = on && s.w_pre ? load_gain(s.w_pre, e, s.dim) : one;
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
        const int j = first + r < (int)a.n ? first + r : (int)a.n - 1;
        row[r] = j < 0 ? 0u : a.rows ? a.rows[j] : (uint32_t)j;
        h[r] = y[r] = v4f{0.f, 0.f, 0.f, 0.f};
        if constexpr (GAINS) y2[r] = add[r] = v4f{0.f, 0.f, 0.f, 0.f};
        if (!on || first + r < 0) continue;
        h[r] = load4(s.x + (size_t)row[r] * s.x_stride + e);
        if (s.y) y[r] = load4(s.y + (size_t)row[r] * s.y_stride + e);
        if constexpr (GAINS) {
            if (s.y2) y2[r] = load4(s.y2 + (size_t)row[r] * s.y_stride + e);
            if (s.add) add[r] = load4(s.add + (size_t)row[r] * s.y_stride + e);
        }
    }
    if (s.experts) {
        const float share = 1.0f / (float)s.top;
        for (uint32_t k = 0; k < s.top; k++) {
            v4f v[R];
#pragma unroll
            for (int r = 0; r < R; r++)
                v[r] = on && first + r >= 0 ? load4(s.experts + (size_t)s.slots[(size_t)row[r] * s.top + k] * s.y_stride + e) : v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int r = 0; r < R; r++) y[r] += v[r] * share;
        }
    }
    float ss[R];
    if constexpr (GAINS) {
        if (has_y) {
            float both[2 * R];
#pragma unroll
            for (int r = 0; r < R; r++) {
                y[r] = mask4(y[r], e, s.dim), y2[r] = mask4(y2[r], e, s.dim);
                both[r] = dot4(y[r], y[r]), both[R + r] = dot4(y2[r], y2[r]);
            }
            block_sums<2 * R, NT>(both, red);
#pragma unroll
            for (int r = 0; r < R; r++) {
                h[r] += y[r] * wp * (s.g_post / sqrtf(both[r] / (float)s.dim + s.eps));
                if (s.y2) h[r] += y2[r] * wp2 * (s.g_post / sqrtf(both[R + r] / (float)s.dim + s.eps));
            }
        }
#pragma unroll
        for (int r = 0; r < R; r++) h[r] += add[r];
    } else if (has_y) {
#pragma unroll
        for (int r = 0; r < R; r++) y[r] = mask4(y[r], e, s.dim), ss[r] = dot4(y[r], y[r]);
        block_sums<R, NT>(ss, red);
#pragma unroll
        for (int r = 0; r < R; r++) h[r] += y[r] * (s.g_post / sqrtf(ss[r] / (float)s.dim + s.eps));
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
        h[r] = mask4(h[r], e, s.dim);
        if (s.x_out && on && r >= own && first + r < (int)a.n) *reinterpret_cast<v4f*>(s.x_out + (size_t)row[r] * s.x_stride + e) = h[r];
    }
    if constexpr (NORM) {
#pragma unroll
        for (int r = 0; r < R; r++) ss[r] = dot4(h[r], h[r]);
        block_sums<R, NT>(ss, red);
#pragma unroll
        for (int r = 0; r < R; r++) h[r] *= s.g_pre / sqrtf(ss[r] / (float)s.dim + s.eps);
        if constexpr (GAINS) {
#pragma unroll
            for (int r = 0; r < R; r++) h[r] *= wn;
        }
    }
}

template <int MODE, bool CONV, bool GAINS, int R, int NT, typename AT>
__global__ __launch_bounds__(NT) void rows_fast_kernel(RowsArgs a) {
    constexpr int HALO = CONV ? kHalo : 0, TILE = R - HALO;
    __shared__ float red[(GAINS ? 2 : 1) * R * (NT / 64)];
    const RowStage& s = a.s;
    const uint32_t e = 4u * threadIdx.x;
    const int j0 = (int)blockIdx.x * TILE;
    v4f w[kHalo + 1], h[R];
    if constexpr (CONV) {
#pragma unroll
        for (int m = 0; m <= kHalo; m++)  // by distance: the newest input is the last tap
            w[m] = m < (int)s.taps && e < s.dim ? mask4(load4(s.conv + (size_t)(s.taps - 1u - m) * s.x_stride + e), e, s.dim) : v4f{0.f, 0.f, 0.f, 0.f};
    }
    stage_tile<MODE == kRowNorm, GAINS, R, NT>(a, j0 - HALO, HALO, h, red);
    if constexpr (MODE == kRowOnly) return;
    if constexpr (CONV) {
        if (j0 == 0) {  // the inputs in front of this portion
#pragma unroll
            for (int r = 0; r < HALO; r++) {
                const int p = (int)a.pos0 + r - HALO;
                h[r] = p >= 0 && HALO - r < (int)s.taps && e < s.dim ? mask4(load4(s.ring + (size_t)((uint32_t)p % s.taps) * s.x_stride + e), e, s.dim)
                                                                      : v4f{0.f, 0.f, 0.f, 0.f};
            }
        }
    }
    if (MODE == kRowNorm && !CONV && a.gate_w) {
        float d[R];
        const uint2 g = e < a.kp ? *reinterpret_cast<const uint2*>(a.gate_w + e) : uint2{0, 0};
        const v4f gw = {__uint_as_float(g.x << 16), __uint_as_float(g.x & 0xffff0000u), __uint_as_float(g.y << 16), __uint_as_float(g.y & 0xffff0000u)};
#pragma unroll
        for (int r = 0; r < R; r++) d[r] = dot4(h[r], gw);
        block_sums<R, NT>(d, red);
        if (threadIdx.x == 0) {
#pragma unroll
            for (int r = 0; r < R; r++)
                if (j0 + r < (int)a.n) a.row_gate[j0 + r] = 1.0f / (1.0f + expf(-d[r]));
        }
    }
#pragma unroll
    for (int r = HALO; r < R; r++) {
        const int j = j0 + r - HALO;
        if (j >= (int)a.n || e >= a.kp) continue;
        v4f v = h[r];
        if constexpr (CONV) {
            v4f c = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int m = kHalo; m >= 0; m--) c += w[m] * h[r - m];
            v += c;
        }
        AT* o = static_cast<AT*>(a.out) + (size_t)j * a.ldo + e;
        if constexpr (MODE == kRowSplit && sizeof(AT) == 2) {
            v4f hi;
#pragma unroll
            for (int i = 0; i < 4; i++) hi[i] = (float)(__bf16)v[i];
            store4(o, hi), store4(o + a.lo_at, v - hi);
        } else {
            store4(o, v);
        }
    }
    if constexpr (CONV) {
        if (j0 == 0) {  // the only workgroup that reads the ring writes it: the portion's last inputs
            v4f tail[kHalo + 1];
            RowsArgs b = a;
            b.s.x_out = nullptr;
            stage_tile<true, GAINS, kHalo + 1, NT>(b, (int)a.n - kHalo - 1, kHalo + 1, tail, red);
#pragma unroll
            for (int r = 0; r <= kHalo; r++) {
                const int j = (int)a.n - kHalo - 1 + r;
                if (j >= 0 && kHalo + 1 - r <= (int)s.taps && e < s.dim)
                    *reinterpret_cast<v4f*>(s.ring + (size_t)((a.pos0 + (uint32_t)j) % s.taps) * s.x_stride + e) = tail[r];
            }
        }
    }
}

template <typename AT>
__global__ __launch_bounds__(256) void embed_activation_kernel(const uint16_t* __restrict__ embed, uint32_t vocab, uint32_t dim, float scale,
                                                               const uint32_t* __restrict__ tokens, float* __restrict__ x, uint32_t x_stride,
                                                               AT* __restrict__ xa, uint32_t ldo, uint32_t kp) {
    const uint32_t t = blockIdx.x, token = tokens[t];
    const uint16_t* row = embed + (size_t)(token < vocab ? token : 0u) * dim;  // the host refuses tokens past the vocabulary
    const uint32_t width = xa ? kp : dim;
    for (uint32_t e = threadIdx.x; e < width; e += 256) {
        const float v = e < dim ? __uint_as_float((uint32_t)row[e] << 16) * scale : 0.0f;
        if (e < dim) x[(size_t)t * x_stride + e] = v;
        if (xa) put(xa + (size_t)t * ldo + e, v);
    }
}

// One row per workgroup, in LDS meanwhile: every part's sum of squares by one wave (few parts: by the whole workgroup).
template <typename AT>
__global__ __launch_bounds__(256) void part_norm_kernel(const float* __restrict__ y, uint32_t ldy, uint32_t dim, uint32_t parts, const float* __restrict__ w,
                                                        float eps, AT* __restrict__ out, uint32_t ldo, uint32_t kp) {
    extern __shared__ __align__(16) float row[];  // [dim] | [parts]
    float* inv = row + dim;
    const uint32_t tid = threadIdx.x;
    const float* src = y + (size_t)blockIdx.x * ldy;
    for (uint32_t e = tid; e < dim; e += 256) row[e] = src[e];
    __syncthreads();
    part_rms(row, dim, parts, eps, inv);
    const uint32_t len = dim / parts;
    for (uint32_t e = tid; e < kp; e += 256) put(out + (size_t)blockIdx.x * ldo + e, e < dim ? row[e] * inv[e / len] * w[e] : 0.0f);
}

// One workgroup per table: counts per expert, their running sums and tiles, then every pair to its entry.  The order of an
// expert's entries is not fixed; no result depends on it.
__global__ __launch_bounds__(256) void route_kernel(const RouteJob* __restrict__ jobs, const uint32_t* __restrict__ tokens, uint32_t n) {
    __shared__ uint32_t count[kRouteMaxExperts], chunk_entries[256], chunk_tiles[256];
    const RouteJob job = jobs[blockIdx.x];
    const uint32_t tid = threadIdx.x, pairs = n * job.top;
    for (uint32_t e = tid; e < job.experts; e += 256) count[e] = 0;
    __syncthreads();
    for (uint32_t p = tid; p < pairs; p += 256) atomicAdd(&count[job.table[(size_t)tokens[p / job.top] * job.top + p % job.top]], 1u);
    __syncthreads();
    const uint32_t per = (job.experts + 255u) / 256u, e0 = tid * per, e1 = e0 + per < job.experts ? e0 + per : job.experts;
    uint32_t entries = 0, tiles = 0;
    for (uint32_t e = e0; e < e1; e++) entries += count[e], tiles += (count[e] + kGroupTileRows - 1u) / kGroupTileRows;
    chunk_entries[tid] = entries, chunk_tiles[tid] = tiles;
    __syncthreads();
    if (tid == 0) {
        uint32_t se = 0, st = 0;
        for (uint32_t i = 0; i < (job.experts + per - 1u) / per; i++) {
            const uint32_t ce = chunk_entries[i], ct = chunk_tiles[i];
            chunk_entries[i] = se, chunk_tiles[i] = st;
            se += ce, st += ct;
        }
        *job.n_tiles = st;
    }
    __syncthreads();
    uint32_t at = chunk_entries[tid], tile = chunk_tiles[tid];
    for (uint32_t e = e0; e < e1; e++) {
        const uint32_t c = count[e];
        for (uint32_t done = 0; done < c; done += kGroupTileRows)
            job.tiles[tile++] = GroupTile{e, at + done, c - done < kGroupTileRows ? c - done : kGroupTileRows};
        count[e] = at;  // now the expert's next free entry
        at += c;
    }
    __syncthreads();
    for (uint32_t p = tid; p < pairs; p += 256) {
        const uint32_t t = p / job.top;
        const uint32_t entry = atomicAdd(&count[job.table[(size_t)tokens[t] * job.top + p % job.top]], 1u);
        job.entry_token[entry] = t;
        job.slot_of[p] = entry;
    }
}

template <int MODE, bool CONV, typename AT>
hipError_t run_rows(const RowsArgs& a, const Launch& L) {
    const uint32_t kp = MODE == kRowOnly ? a.s.dim : a.kp;
    const bool aligned = a.s.x_stride % 4u == 0 && (a.s.y_stride % 4u == 0) && a.ldo % 4u == 0 && a.lo_at % 4u == 0 && kp <= pad_to(a.s.dim, kDensePad) &&
                         pad_to(a.s.dim, kDensePad) <= a.s.x_stride && (!a.s.pending() || pad_to(a.s.dim, kDensePad) <= a.s.y_stride);
    if (aligned && kp <= 4096u && (!CONV || a.s.taps <= (uint32_t)kHalo + 1u)) {
        auto go = [&](auto gains) {
            constexpr bool G = decltype(gains)::value;
            constexpr int R = CONV ? 11 : 4;
            const dim3 grid((a.n + R - (CONV ? kHalo : 0) - 1) / (R - (CONV ? kHalo : 0)));
            if (kp <= 1024u) return launch_kernel(L, kFamOther, rows_fast_kernel<MODE, CONV, G, R, 256, AT>, grid, dim3(256), a);
            if (kp <= 2048u) return launch_kernel(L, kFamOther, rows_fast_kernel<MODE, CONV, G, R, 512, AT>, grid, dim3(512), a);
            return launch_kernel(L, kFamOther, rows_fast_kernel<MODE, CONV, G, CONV ? 7 : 4, 1024, AT>, CONV ? dim3((a.n + 3u) / 4u) : grid, dim3(1024), a);
        };
        if (!a.s.vector_gains()) return go(std::false_type{});
        if constexpr (!CONV) return go(std::true_type{});  // (with a convolution: the general form)
    }
    const uint32_t halo = CONV ? a.s.taps - 1u : 0u;
    uint32_t tile = 8;
    while (tile > 1 && tile / 2 >= halo && (size_t)(tile + halo) * a.s.dim * 4u > 64u * 1024u) tile /= 2;
    if (tile < halo) tile = halo;
    const size_t lds = (size_t)(tile + halo) * a.s.dim * 4u;
    if (lds > kRowsLdsBytes) return hipErrorInvalidValue;
    if (lds > 64u * 1024u) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(rows_kernel<MODE, CONV, AT>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                                 (int)kRowsLdsBytes);
        if (e != hipSuccess) return e;
    }
    return launch_kernel_lds(L, kFamOther, rows_kernel<MODE, CONV, AT>, dim3((a.n + tile - 1) / tile), dim3(256), (uint32_t)lds, a, tile);
}

}  // namespace

uint32_t rows_max_dim(uint32_t taps) {
    const uint32_t halo = taps > 0 ? taps - 1u : 0u;
    return kRowsLdsBytes / 4u / (2u * halo > 1u ? 2u * halo : 1u);
}

hipError_t launch_rows(const RowsArgs& a, int mode, const Launch& L) {
    if (a.n == 0) return hipSuccess;
    const bool conv = a.s.conv != nullptr;
    if (!a.s.x || a.s.dim == 0 || a.s.x_stride < a.s.dim || (mode != kRowOnly && (!a.out || a.kp < a.s.dim || a.ldo < a.kp)) || (conv && (a.rows || !a.s.ring || a.s.taps == 0)) ||
        (mode != kRowNorm && conv) || (mode == kRowOnly && !a.s.x_out) || a.s.x_out == a.s.x || (a.s.y2 && !a.s.y))
        return hipErrorInvalidValue;
    if (mode == kRowNorm) {
        if (conv) return a.f32 ? run_rows<kRowNorm, true, float>(a, L) : run_rows<kRowNorm, true, uint16_t>(a, L);
        return a.f32 ? run_rows<kRowNorm, false, float>(a, L) : run_rows<kRowNorm, false, uint16_t>(a, L);
    }
    if (mode == kRowSplit) return a.f32 ? run_rows<kRowSplit, false, float>(a, L) : run_rows<kRowSplit, false, uint16_t>(a, L);
    return run_rows<kRowOnly, false, float>(a, L);
}

hipError_t launch_part_norm(const float* y, uint32_t ldy, uint32_t n, uint32_t dim, uint32_t parts, const float* w, float eps, void* out, uint32_t ldo, uint32_t kp,
                            bool f32, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (parts == 0 || dim % parts || kp < dim || ldo < kp || ldy < dim || (size_t)(dim + parts) * 4u > 64u * 1024u) return hipErrorInvalidValue;
    const uint32_t lds = (dim + parts) * 4u;
    return f32 ? launch_kernel_lds(L, kFamOther, part_norm_kernel<float>, dim3(n), dim3(256), lds, y, ldy, dim, parts, w, eps, static_cast<float*>(out), ldo, kp)
               : launch_kernel_lds(L, kFamOther, part_norm_kernel<uint16_t>, dim3(n), dim3(256), lds, y, ldy, dim, parts, w, eps, static_cast<uint16_t*>(out), ldo, kp);
}

hipError_t launch_embed_activation(const uint16_t* embed, uint32_t vocab, uint32_t dim, float scale, const uint32_t* tokens, uint32_t n, float* x, uint32_t x_stride, void* xa,
                                   uint32_t ldo, uint32_t kp, bool f32, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (x_stride < dim || (xa && (kp < dim || ldo < kp))) return hipErrorInvalidValue;
    return f32 ? launch_kernel(L, kFamOther, embed_activation_kernel<float>, dim3(n), dim3(256), embed, vocab, dim, scale, tokens, x, x_stride, static_cast<float*>(xa), ldo, kp)
               : launch_kernel(L, kFamOther, embed_activation_kernel<uint16_t>, dim3(n), dim3(256), embed, vocab, dim, scale, tokens, x, x_stride,
                               static_cast<uint16_t*>(xa), ldo, kp);
}

hipError_t launch_route(const RouteJob* d_jobs, uint32_t n_jobs, const uint32_t* tokens, uint32_t n, const Launch& L) {
    if (n_jobs == 0 || n == 0) return hipSuccess;
    return launch_kernel(L, kFamOther, route_kernel, dim3(n_jobs), dim3(256), d_jobs, tokens, n);
}

}  // namespace wick_rocm
