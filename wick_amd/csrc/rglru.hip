// The recurrent block with a real-gated linear recurrent unit (Griffin's): a short causal convolution, two block-diagonal gates and
// a linear recurrence per channel, S_t = a_t S_(t-1) + b_t.  Everything that enters the recurrence is f32.
//
// A prompt runs the gates as one batched product (launch_gemm_gates) and the recurrence as a scan in chunks of tokens: every
// (chunk, channel) first reduces its tokens to one affine map, then starts from the maps of the chunks before it.  A decode step
// does everything between the block's projections in one launch.
#include "wick_rocm_dense.h"
#include "short_conv.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

constexpr uint32_t kScanChunk = 32;

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(uint16_t* p, float v) { *p = __builtin_bit_cast(uint16_t, (__bf16)v); }

// u as f32 rows and in the activation type of the gates' product (bfloat16: two terms).
template <typename AT>
struct ConvToGates {
    float* u;
    AT* ua;
    uint32_t channels, block, lda;
    __device__ void operator()(uint32_t ch, uint32_t t0, const float (&v)[kConvTokens], uint32_t count) const {
        const uint32_t terms = sizeof(AT) == 2 ? 2u : 1u;
        AT* o = ua + (size_t)(ch / block) * terms * block + ch % block + (size_t)t0 * lda;
#pragma unroll
        for (uint32_t i = 0; i < kConvTokens; i++, o += lda) {
            if (i >= count) break;
            u[(size_t)(t0 + i) * channels + ch] = v[i];
            if constexpr (sizeof(AT) == 2) {
                const float hi = (float)(__bf16)v[i];
                put(o, hi), put(o + block, v[i] - hi);
            } else {
                put(o, v[i]);
            }
        }
    }
};

// Scratch: [chunks][channels] products of a, the same of the chunk's own result, [channels] the state the portion starts from.
// The first chunk's result already contains that state.
__global__ __launch_bounds__(256) void scan_chunks_kernel(const float* __restrict__ a, const float* __restrict__ b, const float* __restrict__ state,
                                                          uint32_t n, uint32_t channels, uint32_t pos0, float* __restrict__ scratch) {
    const uint32_t ch = blockIdx.x * 256u + threadIdx.x, c = blockIdx.y, chunks = gridDim.y;
    if (ch >= channels) return;
    float prod = 1.0f, s = 0.0f;
    if (c == 0) {
        s = pos0 > 0 ? state[ch] : 0.0f;
        scratch[(size_t)2 * chunks * channels + ch] = s;
    }
    const uint32_t t0 = c * kScanChunk, nt = n - t0 < kScanChunk ? n - t0 : kScanChunk;
    for (uint32_t i = 0; i < nt; i += 16) {
        float av[16], bv[16];
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const size_t at = (size_t)(t0 + (i + j < nt ? i + j : nt - 1u)) * channels + ch;
            av[j] = a[at], bv[j] = b[at];
        }
#pragma unroll
        for (int j = 0; j < 16; j++)
            if (i + j < nt) prod *= av[j], s = av[j] * s + bv[j];
    }
    scratch[(size_t)c * channels + ch] = prod;
    scratch[(size_t)(chunks + c) * channels + ch] = s;
}

template <typename AT>
__global__ __launch_bounds__(256) void scan_apply_kernel(const float* __restrict__ a, const float* __restrict__ b, const float* __restrict__ y,
                                                         uint32_t ldy, float* __restrict__ state, uint32_t n, uint32_t channels,
                                                         const float* __restrict__ scratch, AT* __restrict__ out, uint32_t ldo, uint32_t kp) {
    const uint32_t ch = blockIdx.x * 256u + threadIdx.x, c = blockIdx.y, chunks = gridDim.y;
    if (ch >= kp) return;
    const uint32_t t0 = c * kScanChunk, nt = n - t0 < kScanChunk ? n - t0 : kScanChunk;
    if (ch >= channels) {
        for (uint32_t i = 0; i < nt; i++) put(out + (size_t)(t0 + i) * ldo + ch, 0.0f);
        return;
    }
    float s = scratch[(size_t)(c == 0 ? 2u * chunks : chunks) * channels + ch];  // the start of the portion / the end of chunk 0
    for (uint32_t q0 = 1; q0 < c; q0 += 8) {
        float av[8], bv[8];
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const uint32_t q = q0 + j < c ? q0 + j : c - 1u;
            av[j] = scratch[(size_t)q * channels + ch], bv[j] = scratch[(size_t)(chunks + q) * channels + ch];
        }
#pragma unroll
        for (int j = 0; j < 8; j++)
            if (q0 + j < c) s = av[j] * s + bv[j];
    }
    for (uint32_t i = 0; i < nt; i += 16) {
        float av[16], bv[16], yv[16];
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const uint32_t t = t0 + (i + j < nt ? i + j : nt - 1u);
            av[j] = a[(size_t)t * channels + ch], bv[j] = b[(size_t)t * channels + ch], yv[j] = y[(size_t)t * ldy + ch];
        }
#pragma unroll
        for (int j = 0; j < 16; j++)
            if (i + j < nt) {
                s = av[j] * s + bv[j];
                put(out + (size_t)(t0 + i + j) * ldo + ch, s * yv[j]);
            }
    }
    if (c + 1 == chunks) state[ch] = s;
}

// Workgroup (block, part): the convolution of the whole block (every gate row needs it), then kStepPart channels of it, a group of
// LPR lanes per channel.  The first part of a block writes the block's newest input to the ring, into a slot nobody reads.
constexpr uint32_t kStepPart = 32;
constexpr uint32_t kStepMaxBlock = 4096;

template <int LPR>
__global__ __launch_bounds__(256) void recurrent_step_kernel(RecurrentStep a) {
    extern __shared__ __align__(16) float u[];
    const uint32_t parts = a.block / kStepPart, blk = blockIdx.x / parts, part = blockIdx.x % parts;
    const uint32_t tid = threadIdx.x, pos = *a.d_pos, c0 = blk * a.block;
    const uint32_t l = tid % LPR, grp = tid / LPR;
    const uint16_t* w = a.gates.d + (size_t)blk * a.gates.stride;
    auto row_of = [&](uint32_t f) { return w + (size_t)((f >> 4) * 32u + (f & 15u)) * a.gates.kp; };
    // requested before the convolution whose result they meet
    const uint16_t* row0 = row_of(part * kStepPart + grp);
    const uint32_t at0 = 8u * l < a.block ? 8u * l : 0u;
    const uint4 q0 = *reinterpret_cast<const uint4*>(row0 + at0), p0 = *reinterpret_cast<const uint4*>(row0 + (size_t)16 * a.gates.kp + at0);
    // ... and so is what the first pass of channels needs behind it
    const uint32_t ch0 = c0 + part * kStepPart + grp;
    const float rb0 = a.r_bias[ch0], ib0 = a.i_bias[ch0], rate0 = a.rate[ch0], s0 = a.state[ch0], y0 = a.proj[ch0];
    for (uint32_t i = tid; i < a.block; i += 256) {
        const uint32_t ch = c0 + i;
        const float now = a.proj[a.channels + ch];
        float v = 0.0f;
        if (a.taps <= 4u) {  // every tap's loads in flight together
            float w[4], in[4];
#pragma unroll
            for (uint32_t m = 1; m < 4; m++) {
                const bool on = m < a.taps;
                w[m] = on ? a.conv_w[(size_t)(a.taps - 1u - m) * a.channels + ch] : 0.0f;
                in[m] = on && pos >= m ? a.ring[(size_t)((pos - m) % a.taps) * a.channels + ch] : 0.0f;
            }
#pragma unroll
            for (uint32_t m = 3; m > 0; m--) v += w[m] * in[m];
        } else {
            for (uint32_t m = a.taps - 1u; m > 0; m--)
                v += a.conv_w[(size_t)(a.taps - 1u - m) * a.channels + ch] * (pos >= m ? a.ring[(size_t)((pos - m) % a.taps) * a.channels + ch] : 0.0f);
        }
        v += a.conv_w[(size_t)(a.taps - 1u) * a.channels + ch] * now;
        u[i] = v + a.conv_bias[ch];
        if (part == 0) a.ring[(size_t)(pos % a.taps) * a.channels + ch] = now;
    }
    __syncthreads();
    for (uint32_t f0 = 0; f0 < kStepPart; f0 += 256u / LPR) {
        const uint32_t f = part * kStepPart + f0 + grp;  // channel of the block; LPR >= 8: a pass covers at most kStepPart channels
        const uint16_t* rw = row_of(f);
        const uint16_t* iw = rw + (size_t)16 * a.gates.kp;
        float r = 0.0f, g = 0.0f;
        for (uint32_t at = 8u * l; at < a.block; at += 8u * LPR) {
            const bool first = f0 == 0 && at == 8u * l;
            const uint4 q = first ? q0 : *reinterpret_cast<const uint4*>(rw + at), p = first ? p0 : *reinterpret_cast<const uint4*>(iw + at);
            const uint32_t qv[4] = {q.x, q.y, q.z, q.w}, pv[4] = {p.x, p.y, p.z, p.w};
#pragma unroll
            for (int k = 0; k < 4; k++) {
                r = fmaf(__uint_as_float(qv[k] << 16), u[at + 2 * k], r), r = fmaf(__uint_as_float(qv[k] & 0xffff0000u), u[at + 2 * k + 1], r);
                g = fmaf(__uint_as_float(pv[k] << 16), u[at + 2 * k], g), g = fmaf(__uint_as_float(pv[k] & 0xffff0000u), u[at + 2 * k + 1], g);
            }
        }
        r = group_sum<LPR>(r), g = group_sum<LPR>(g);
        if (l == 0) {
            const uint32_t ch = c0 + f;
            const bool first = f0 == 0;
            r = 1.0f / (1.0f + expf(-(r + (first ? rb0 : a.r_bias[ch])))), g = 1.0f / (1.0f + expf(-(g + (first ? ib0 : a.i_bias[ch]))));
            const float log_a = r * (first ? rate0 : a.rate[ch]), decay = expf(log_a);
            const float s = decay * (pos == 0 ? 0.0f : first ? s0 : a.state[ch]) + sqrtf(-expm1f(2.0f * log_a)) * (g * u[f]);
            a.state[ch] = s;
            a.out[ch] = s * (first ? y0 : a.proj[ch]);
        }
    }
}

}  // namespace

hipError_t launch_recurrent_conv(const RecurrentConv& a, uint32_t n, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (a.taps == 0 || a.taps > kConvTokens || a.block == 0 || a.channels % a.block || a.lda < a.channels * (a.f32 ? 1u : 2u)) return hipErrorInvalidValue;
    const ShortConv c{a.proj + a.x_at, a.ldp, a.channels, a.taps, a.pos0, a.w, a.bias, a.ring};
    return a.f32 ? launch_short_conv(c, n, n, ConvToGates<float>{a.u, static_cast<float*>(a.ua), a.channels, a.block, a.lda}, L)
                 : launch_short_conv(c, n, n, ConvToGates<uint16_t>{a.u, static_cast<uint16_t*>(a.ua), a.channels, a.block, a.lda}, L);
}

size_t recurrent_scan_scratch_floats(uint32_t n, uint32_t channels) { return ((size_t)2 * ((n + kScanChunk - 1u) / kScanChunk) + 1u) * channels; }

hipError_t launch_recurrent_scan(const float* a, const float* b, const float* y, uint32_t ldy, float* state, uint32_t n, uint32_t channels, uint32_t pos0,
                                 void* out, uint32_t ldo, uint32_t kp, bool f32, float* scratch, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (kp < channels || ldo < kp || ldy < channels) return hipErrorInvalidValue;
    const uint32_t chunks = (n + kScanChunk - 1u) / kScanChunk;
    hipError_t e = launch_kernel(L, kFamOther, scan_chunks_kernel, dim3((channels + 255u) / 256u, chunks), dim3(256), a, b, static_cast<const float*>(state), n,
                                 channels, pos0, scratch);
    if (e != hipSuccess) return e;
    const dim3 grid((kp + 255u) / 256u, chunks);
    const float* sc = scratch;
    return f32 ? launch_kernel(L, kFamOther, scan_apply_kernel<float>, grid, dim3(256), a, b, y, ldy, state, n, channels, sc, static_cast<float*>(out), ldo, kp)
               : launch_kernel(L, kFamOther, scan_apply_kernel<uint16_t>, grid, dim3(256), a, b, y, ldy, state, n, channels, sc,
                               static_cast<uint16_t*>(out), ldo, kp);
}

hipError_t launch_recurrent_step(const RecurrentStep& a, const Launch& L) {
    if (a.block == 0 || a.block % kDensePad || a.block > kStepMaxBlock || a.blocks * a.block != a.channels || a.gates.mp != 2u * a.block ||
        a.gates.kp < a.block || a.taps == 0 || !a.d_pos)
        return hipErrorInvalidValue;
    const dim3 grid(a.blocks * (a.block / kStepPart));
    const uint32_t lds = a.block * 4u;
    if (a.block <= 64u) return launch_kernel_lds(L, kFamGemv, recurrent_step_kernel<8>, grid, dim3(256), lds, a);
    if (a.block <= 128u) return launch_kernel_lds(L, kFamGemv, recurrent_step_kernel<16>, grid, dim3(256), lds, a);
    if (a.block <= 256u) return launch_kernel_lds(L, kFamGemv, recurrent_step_kernel<32>, grid, dim3(256), lds, a);
    return launch_kernel_lds(L, kFamGemv, recurrent_step_kernel<64>, grid, dim3(256), lds, a);
}

}  // namespace wick_rocm
