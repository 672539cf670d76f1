// A prompt's causal depthwise convolution over time in front of a recurrence, with what happens to its results as a functor.
// The last `taps` inputs of a sequence live in a ring: position p in slot p % taps.  Not installed.
#pragma once

#include <type_traits>

#include "wick_rocm_internal.h"

namespace wick_rocm {

constexpr uint32_t kConvTokens = 8;  // tokens per thread; at least taps - 1

struct ShortConv {
    const float* x;          // [n][ldx]: the inputs
    uint32_t ldx, channels, taps, pos0;
    const float *w, *bias;   // [taps][channels], [channels]
    float* ring;             // [taps][channels]
};

// One thread: one channel, kConvTokens tokens, their inputs and the ones in front of them in registers (FAST: up to four taps).
// Only the threads of the first tokens read the ring, and they alone write it, after their reads.  sink(channel, first token, results,
// how many of them are tokens of the portion).
template <bool FAST, class Sink>
__global__ __launch_bounds__(256) void short_conv_kernel(ShortConv a, uint32_t n, Sink sink) {
    constexpr int BACK = FAST ? 3 : (int)kConvTokens;
    const uint32_t ch = blockIdx.x * 256u + threadIdx.x, t0 = blockIdx.y * kConvTokens;
    if (ch >= a.channels) return;
    const float* x = a.x + ch;
    const float bias = a.bias[ch];
    float in[BACK + (int)kConvTokens], w[BACK + 1], out[kConvTokens];  // w by distance: the newest input is the last tap
#pragma unroll
    for (int i = 0; i < BACK + (int)kConvTokens; i++) {
        const int t = (int)t0 + i - BACK, p = (int)a.pos0 + t;
        in[i] = 0.0f;
        if (t >= 0) in[i] = x[(size_t)(t < (int)n ? t : (int)n - 1) * a.ldx];
        else if (p >= 0 && BACK - i < (int)a.taps) in[i] = a.ring[(size_t)((uint32_t)p % a.taps) * a.channels + ch];
    }
#pragma unroll
    for (int m = 0; m <= BACK; m++) w[m] = m < (int)a.taps ? a.w[(size_t)(a.taps - 1u - m) * a.channels + ch] : 0.0f;
#pragma unroll
    for (int i = 0; i < (int)kConvTokens; i++) {
        float v = 0.0f;
#pragma unroll
        for (int m = BACK; m >= 0; m--) v += w[m] * in[i + BACK - m];
        out[i] = v + bias;
    }
    sink(ch, t0, out, t0 >= n ? 0u : n - t0 < kConvTokens ? n - t0 : kConvTokens);
    if (blockIdx.y == 0)
        for (uint32_t t = n > a.taps ? n - a.taps : 0u; t < n; t++) a.ring[(size_t)((a.pos0 + t) % a.taps) * a.channels + ch] = x[(size_t)t * a.ldx];
}

// rows: tokens the sink is called for (n, or more when it pads).
template <class Sink>
hipError_t launch_short_conv(const ShortConv& a, uint32_t n, uint32_t rows, const Sink& sink, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (a.taps == 0 || a.taps > kConvTokens || rows < n) return hipErrorInvalidValue;
    const dim3 grid((a.channels + 255u) / 256u, (rows + kConvTokens - 1u) / kConvTokens);
    return a.taps <= 4u ? launch_kernel(L, kFamOther, short_conv_kernel<true, Sink>, grid, dim3(256), a, n, sink)
                        : launch_kernel(L, kFamOther, short_conv_kernel<false, Sink>, grid, dim3(256), a, n, sink);
}

}  // namespace wick_rocm
