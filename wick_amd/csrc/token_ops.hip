// The two ends of a step that every model shares: a token's embedding row as f32 and the greedy pick over the logits, with the
// device-side token / position that let a captured graph of the step be replayed.  Arithmetic follows the reference's CPU
// operations (wick/src/model/lfm2.rs:621-643, wick/src/sampler.rs:7-19), bit for bit.
#include "wick_rocm_device.h"
#include "wick_rocm_internal.h"

namespace wick_rocm {

namespace {

// ---- embedding row -------------------------------------------------------------------
// dequantize_row_into (wick/src/model/lfm2.rs:621-643) for Q4_0 / Q8_0 (quant.rs:78-90, 154-161) and
// Q6_K (quant.rs:380-412: d * sc * q left to right), and plain BF16 rows: bit-exact.
__device__ __forceinline__ float dequant_element(const uint8_t* __restrict__ w, int type, uint32_t row, uint32_t k, uint32_t e) {
    if (type == kTypeBF16) return __uint_as_float((uint32_t)reinterpret_cast<const uint16_t*>(w)[(size_t)row * k + e] << 16);
    if (type == kTypeQ6_K) {
        const uint8_t* blk = w + ((size_t)row * (k >> 8) + (e >> 8)) * kQ6KBlockBytes;
        const uint32_t i = e & 255u, n = i >> 7, j = (i >> 5) & 3u, l = i & 31u;
        const uint32_t lo = (blk[64 * n + 32 * (j & 1u) + l] >> (4 * (j >> 1))) & 15u;
        const uint32_t hi = (blk[128 + 32 * n + l] >> (2 * j)) & 3u;
        const int q = (int)(lo | (hi << 4)) - 32;
        const float d = f16_bits_to_f32((uint32_t)blk[208] | ((uint32_t)blk[209] << 8));
        const float sc = (float)(int)(int8_t)blk[192 + (i >> 4)];
        return __fmul_rn(__fmul_rn(d, sc), (float)q);
    }
    if (type == kTypeQ4_0) {
        const uint8_t* blk = w + ((size_t)row * (k >> 5) + (e >> 5)) * kQ4BlockBytes;
        const uint32_t i = e & 31u;
        const uint32_t byte = blk[2 + (i & 15u)];
        const int q = (int)((i < 16u) ? (byte & 15u) : (byte >> 4)) - 8;
        return __fmul_rn((float)q, f16_bits_to_f32((uint32_t)blk[0] | ((uint32_t)blk[1] << 8)));
    }
    const uint8_t* blk = w + ((size_t)row * (k >> 5) + (e >> 5)) * kQ8BlockBytes;
    return __fmul_rn((float)(int)(int8_t)blk[2 + (e & 31u)], f16_bits_to_f32((uint32_t)blk[0] | ((uint32_t)blk[1] << 8)));
}

__global__ __launch_bounds__(256) void embed_row_kernel(const uint8_t* __restrict__ w, int type, uint32_t m, uint32_t k, uint32_t token,
                                                        const uint32_t* __restrict__ d_token, float* __restrict__ out) {
    const uint32_t row = d_token ? *d_token : token;
    if (row >= m) return;  // the host checks a by-value token; a device-side token out of range leaves `out` untouched
    for (uint32_t e = blockIdx.x * blockDim.x + threadIdx.x; e < k; e += gridDim.x * blockDim.x) out[e] = dequant_element(w, type, row, k, e);
}

// The rows of a whole prompt: out[j][k] = row d_tokens[j] (blockIdx.y = j).
__global__ __launch_bounds__(256) void embed_rows_kernel(const uint8_t* __restrict__ w, int type, uint32_t m, uint32_t k,
                                                         const uint32_t* __restrict__ d_tokens, float* __restrict__ out) {
    const uint32_t row = d_tokens[blockIdx.y];
    if (row >= m) return;
    float* o = out + (size_t)blockIdx.y * k;
    for (uint32_t e = blockIdx.x * blockDim.x + threadIdx.x; e < k; e += gridDim.x * blockDim.x) o[e] = dequant_element(w, type, row, k, e);
}

// ---- greedy pick ----------------------------------------------------------------------
// cpu_argmax (wick/src/sampler.rs:7-19): NaN counts as -inf, values order by f32::total_cmp, the LAST of
// equal maxima wins; bit-exact.  Two small launches (64 blocks, then one wave over their partial keys): a single
// block would spend 20 us walking a 65536-entry vocabulary.  Optionally publishes the pick as the next step's
// token and advances the device-side position.

constexpr uint32_t kArgmaxBlocks = 64;

// Stage 1: every block leaves the best key of its slice (float4 loads, all of a thread's loads in flight at once).
__global__ __launch_bounds__(256) void argmax_partial_kernel(const float* __restrict__ x, uint32_t n, unsigned long long* __restrict__ partial) {
    __shared__ unsigned long long red[4];
    unsigned long long best = 0ull;  // below every real key
    const uint32_t quads = n >> 2, stride = gridDim.x * 256u;
    for (uint32_t q0 = blockIdx.x * 256u + threadIdx.x; q0 < quads; q0 += 4u * stride) {
        float4 v[4];
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t q = q0 + j * stride;
            v[j] = reinterpret_cast<const float4*>(x)[q < quads ? q : q0];  // clamped: a repeated quad cannot change the maximum
        }
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t q = q0 + j * stride;
            const uint32_t i = 4u * (q < quads ? q : q0);
            const unsigned long long k0 = argmax_key(v[j].x, i), k1 = argmax_key(v[j].y, i + 1), k2 = argmax_key(v[j].z, i + 2),
                                     k3 = argmax_key(v[j].w, i + 3);
            const unsigned long long a = k0 > k1 ? k0 : k1, b = k2 > k3 ? k2 : k3, c = a > b ? a : b;
            best = c > best ? c : best;
        }
    }
    if (blockIdx.x == 0 && threadIdx.x < (n & 3u)) {  // the last n % 4 elements
        const uint32_t i = (n & ~3u) + threadIdx.x;
        const unsigned long long k = argmax_key(x[i], i);
        best = k > best ? k : best;
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
        const unsigned long long o = __shfl_xor(best, off, 64);
        best = o > best ? o : best;
    }
    if ((threadIdx.x & 63u) == 0) red[threadIdx.x >> 6] = best;
    __syncthreads();
    if (threadIdx.x == 0) {
        const unsigned long long a = red[0] > red[1] ? red[0] : red[1], b = red[2] > red[3] ? red[2] : red[3];
        partial[blockIdx.x] = a > b ? a : b;
    }
}

// Stage 2: one workgroup (one wave when there are at most 64 keys and nothing to look up) merges the partial keys and
// publishes the pick.
// An embedding to look the next step's input up in (w null: none): row `token` of w as k floats into `out`.
struct EmbedArgs {
    const uint8_t* w;
    float* out;
    int type;
    uint32_t m, k;
    float scale;  // of a looked-up row
};

// Row `row` of the embedding into emb.out by the calling workgroup, four elements per thread at a time: their loads are all issued
// before the first store (the stores could alias the loads as far as the compiler knows, which would chain the round trips).
__device__ __forceinline__ void embed_row_batched(const EmbedArgs& emb, uint32_t row) {
    for (uint32_t e0 = threadIdx.x; e0 < emb.k; e0 += 4u * blockDim.x) {
        float v[4];
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t e = e0 + j * blockDim.x;
            v[j] = dequant_element(emb.w, emb.type, row, emb.k, e < emb.k ? e : e0);
        }
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t e = e0 + j * blockDim.x;
            if (e < emb.k) emb.out[e] = __fmul_rn(v[j], emb.scale);
        }
    }
}

__global__ __launch_bounds__(256) void argmax_final_kernel(const unsigned long long* __restrict__ partial, uint32_t blocks, uint32_t n,
                                                           uint32_t* __restrict__ out, uint32_t* __restrict__ d_token, uint32_t* __restrict__ d_pos,
                                                           uint32_t* __restrict__ d_history, uint32_t history_len, EmbedArgs emb) {
    __shared__ uint32_t picked;
    __shared__ unsigned long long red[4];
    const uint32_t waves = blockDim.x >> 6;  // 1 (at most 64 partial keys) or 4
    unsigned long long best = 0ull;
    for (uint32_t i0 = threadIdx.x; i0 < blocks; i0 += 8u * blockDim.x) {  // eight keys per thread in flight (one round trip for <= 2048 keys)
        unsigned long long k[8];
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const uint32_t i = i0 + j * blockDim.x;
            k[j] = partial[i < blocks ? i : i0];  // clamped: a repeated key cannot change the maximum
        }
#pragma unroll
        for (int j = 0; j < 8; j++) best = k[j] > best ? k[j] : best;
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
        const unsigned long long o = __shfl_xor(best, off, 64);
        best = o > best ? o : best;
    }
    if (waves > 1) {
        if ((threadIdx.x & 63u) == 0) red[threadIdx.x >> 6] = best;
        __syncthreads();
        if (threadIdx.x == 0) {
            const unsigned long long a = red[0] > red[1] ? red[0] : red[1], b = red[2] > red[3] ? red[2] : red[3];
            best = a > b ? a : b;
        }
    }
    if (threadIdx.x == 0) {
        const uint32_t pick = n ? (uint32_t)(best & 0xffffffffull) : 0u;
        picked = pick;
        out[0] = pick;
        if (d_token) *d_token = pick;
        if (d_pos) {
            const uint32_t pos = *d_pos;
            if (d_history && pos < history_len) d_history[pos] = pick;  // the pick made after the token at `pos`
            *d_pos = pos + 1u;
        }
    }
    if (!emb.w) return;
    __syncthreads();
    const uint32_t pick = picked;  // the pick is the next step's token: its embedding row is that step's input
    if (pick < emb.m) embed_row_batched(emb, pick);
}

// Sets the device-side token / position of the next step (either may be null) and, when an embedding is given, looks
// the token's row up as that step's input.
__global__ __launch_bounds__(256) void set_step_kernel(uint32_t* d_token, uint32_t token, uint32_t* d_pos, uint32_t pos, EmbedArgs emb) {
    if (threadIdx.x == 0) {
        if (d_token) *d_token = token;
        if (d_pos) *d_pos = pos;
    }
    if (emb.w && token < emb.m) embed_row_batched(emb, token);
}

__global__ void advance_pos_kernel(uint32_t* d_pos) {
    if (threadIdx.x == 0 && blockIdx.x == 0) *d_pos = *d_pos + 1u;
}

}  // namespace

hipError_t launch_embed_row(const uint8_t* d_w, int type, uint32_t m, uint32_t k, uint32_t token, const uint32_t* d_token, float* d_out,
                            const Launch& L) {
    const uint32_t blocks = (k + 255u) / 256u;
    return launch_kernel(L, kFamOther, embed_row_kernel, dim3(blocks < 64u ? blocks : 64u), dim3(256), d_w, type, m, k, token, d_token, d_out);
}

hipError_t launch_embed_rows(const uint8_t* d_w, int type, uint32_t m, uint32_t k, const uint32_t* d_tokens, uint32_t n, float* d_out,
                             const Launch& L) {
    if (n == 0) return hipSuccess;
    const uint32_t blocks = (k + 255u) / 256u;
    return launch_kernel(L, kFamOther, embed_rows_kernel, dim3(blocks < 16u ? blocks : 16u, n), dim3(256), d_w, type, m, k, d_tokens, d_out);
}

hipError_t launch_argmax(const float* d_x, uint32_t n, unsigned long long* d_partial, uint32_t* d_out, uint32_t* d_token, uint32_t* d_pos,
                         uint32_t* d_history, uint32_t history_len, const Launch& L, const uint8_t* d_embd, int embd_type, uint32_t embd_m,
                         uint32_t embd_k, float* d_embd_out, float embd_scale) {
    const uint32_t blocks = n >= 4096u ? kArgmaxBlocks : 1u;
    hipError_t e = launch_kernel(L, kFamOther, argmax_partial_kernel, dim3(blocks), dim3(256), d_x, n, d_partial);
    if (e != hipSuccess) return e;
    return launch_argmax_final(d_partial, blocks, n, d_out, d_token, d_pos, d_history, history_len, L, d_embd, embd_type, embd_m, embd_k, d_embd_out,
                               embd_scale);
}

hipError_t launch_argmax_final(const unsigned long long* d_partial, uint32_t n_partials, uint32_t n, uint32_t* d_out, uint32_t* d_token, uint32_t* d_pos,
                               uint32_t* d_history, uint32_t history_len, const Launch& L, const uint8_t* d_embd, int embd_type, uint32_t embd_m,
                               uint32_t embd_k, float* d_embd_out, float embd_scale) {
    const EmbedArgs emb{d_embd_out ? d_embd : nullptr, d_embd_out, embd_type, embd_m, embd_k, embd_scale};
    return launch_kernel(L, kFamOther, argmax_final_kernel, dim3(1), dim3(emb.w || n_partials > 64u ? 256 : 64), d_partial, n_partials, n, d_out, d_token,
                         d_pos, d_history, history_len, emb);
}

hipError_t launch_set_step(uint32_t* d_token, uint32_t token, uint32_t* d_pos, uint32_t pos, const Launch& L, const uint8_t* d_embd, int embd_type,
                           uint32_t embd_m, uint32_t embd_k, float* d_embd_out, float embd_scale) {
    const EmbedArgs emb{d_embd_out ? d_embd : nullptr, d_embd_out, embd_type, embd_m, embd_k, embd_scale};
    return launch_kernel(L, kFamOther, set_step_kernel, dim3(1), dim3(256), d_token, token, d_pos, pos, emb);
}

hipError_t launch_advance_pos(uint32_t* d_pos, const Launch& L) {
    return launch_kernel(L, kFamOther, advance_pos_kernel, dim3(1), dim3(64), d_pos);
}

}  // namespace wick_rocm
