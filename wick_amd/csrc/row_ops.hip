// Rows of a prompt between the matrix products: the residual update with its norms, the input convolution, embedding rows and the
// grouping of tokens by expert.  Everything is computed in f32; rows leave in the activation type of the next product.
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

constexpr uint32_t kRowsLdsBytes = 160u * 1024u;

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(uint16_t* p, float v) { *p = __builtin_bit_cast(uint16_t, (__bf16)v); }

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

// One row by the calling wave: dst[0 .. dim) = x + g_post y / rms(y), normed when NORM.  dst may be LDS or global memory; a lane
// only re-reads what it wrote itself.
template <bool NORM>
__device__ __forceinline__ void stage_row(const RowStage& s, uint32_t t, float* dst, float* x_out) {
    const uint32_t lane = threadIdx.x & 63u;
    const float* x = s.x + (size_t)t * s.x_stride;
    const bool has_y = s.y || s.experts;
    float sy = 0.0f;
    if (has_y) {
        float ss = 0.0f;
        for (uint32_t e = lane; e < s.dim; e += 64) {
            const float v = row_y(s, t, e);
            ss += v * v;
        }
        sy = s.g_post / sqrtf(wave_sum_f32(ss) / (float)s.dim + s.eps);
    }
    float ss = 0.0f;
    for (uint32_t e = lane; e < s.dim; e += 64) {
        const float v = has_y ? x[e] + row_y(s, t, e) * sy : x[e];
        dst[e] = v;
        if (x_out) x_out[e] = v;
        ss += v * v;
    }
    if constexpr (NORM) {
        const float sx = s.g_pre / sqrtf(wave_sum_f32(ss) / (float)s.dim + s.eps);
        for (uint32_t e = lane; e < s.dim; e += 64) dst[e] *= sx;
    }
}

// A workgroup takes `tile` consecutive rows; with a convolution it also stages the taps - 1 rows in front of them (from its own
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
            const float* past = p >= 0 ? s.ring + (size_t)((uint32_t)p % s.taps) * dim : nullptr;
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
                    for (uint32_t k = 0; k < s.taps; k++) c += s.conv[(size_t)k * dim + e] * hrow[(size_t)(r + k) * dim + e];
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
        for (uint32_t j = first + wave; j < a.n; j += 4) stage_row<true>(s, j, s.ring + (size_t)((a.pos0 + j) % s.taps) * dim, nullptr);
    }
}

template <typename AT>
__global__ __launch_bounds__(256) void embed_activation_kernel(const uint16_t* __restrict__ embed, uint32_t vocab, uint32_t dim,
                                                               const uint32_t* __restrict__ tokens, float* __restrict__ x, uint32_t x_stride,
                                                               AT* __restrict__ xa, uint32_t ldo, uint32_t kp) {
    const uint32_t t = blockIdx.x, token = tokens[t];
    const uint16_t* row = embed + (size_t)(token < vocab ? token : 0u) * dim;  // the host refuses tokens past the vocabulary
    const uint32_t width = xa ? kp : dim;
    for (uint32_t e = threadIdx.x; e < width; e += 256) {
        const float v = e < dim ? __uint_as_float((uint32_t)row[e] << 16) : 0.0f;
        if (e < dim) x[(size_t)t * x_stride + e] = v;
        if (xa) put(xa + (size_t)t * ldo + e, v);
    }
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
        for (uint32_t i = 0; i < 256; i++) {
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
        (mode != kRowNorm && conv) || (mode == kRowOnly && !a.s.x_out) || a.s.x_out == a.s.x)
        return hipErrorInvalidValue;
    if (mode == kRowNorm) {
        if (conv) return a.f32 ? run_rows<kRowNorm, true, float>(a, L) : run_rows<kRowNorm, true, uint16_t>(a, L);
        return a.f32 ? run_rows<kRowNorm, false, float>(a, L) : run_rows<kRowNorm, false, uint16_t>(a, L);
    }
    if (mode == kRowSplit) return a.f32 ? run_rows<kRowSplit, false, float>(a, L) : run_rows<kRowSplit, false, uint16_t>(a, L);
    return run_rows<kRowOnly, false, float>(a, L);
}

hipError_t launch_embed_activation(const uint16_t* embed, uint32_t vocab, uint32_t dim, const uint32_t* tokens, uint32_t n, float* x, uint32_t x_stride, void* xa,
                                   uint32_t ldo, uint32_t kp, bool f32, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (x_stride < dim || (xa && (kp < dim || ldo < kp))) return hipErrorInvalidValue;
    return f32 ? launch_kernel(L, kFamOther, embed_activation_kernel<float>, dim3(n), dim3(256), embed, vocab, dim, tokens, x, x_stride, static_cast<float*>(xa), ldo, kp)
               : launch_kernel(L, kFamOther, embed_activation_kernel<uint16_t>, dim3(n), dim3(256), embed, vocab, dim, tokens, x, x_stride,
                               static_cast<uint16_t*>(xa), ldo, kp);
}

hipError_t launch_route(const RouteJob* d_jobs, uint32_t n_jobs, const uint32_t* tokens, uint32_t n, const Launch& L) {
    if (n_jobs == 0 || n == 0) return hipSuccess;
    return launch_kernel(L, kFamOther, route_kernel, dim3(n_jobs), dim3(256), d_jobs, tokens, n);
}

}  // namespace wick_rocm
