// Device code of one token through a state-space duality block, shared by the launches it appears in.  Not installed.
#pragma once

#include "short_conv.h"
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));

constexpr uint32_t kRows = 16;  // state rows (value coordinates) of a workgroup in a step / scan: 16 lanes each

__device__ __forceinline__ float siluf(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

struct SsdStepArgs {
    SsdShape s;
    SsdWeights w;
    SsdProj p;
    float *ring, *state, *out;
    const uint32_t* d_pos;
};

// The convolution of one channel at the newest position, then silu.
__device__ __forceinline__ float conv_now(const SsdStepArgs& a, uint32_t ch, uint32_t pos, float now) {
    const uint32_t C = a.s.channels(), taps = a.s.taps;
    float v = 0.0f;
    if (taps <= 4u) {  // every tap's loads in flight together
        float w[4], in[4];
#pragma unroll
        for (uint32_t m = 1; m < 4; m++) {
            const bool on = m < taps;
            w[m] = on ? a.w.conv[(size_t)(taps - 1u - m) * C + ch] : 0.0f;
            in[m] = on && pos >= m ? a.ring[(size_t)((pos - m) % taps) * C + ch] : 0.0f;
        }
#pragma unroll
        for (uint32_t m = 3; m > 0; m--) v += w[m] * in[m];
    } else {
        for (uint32_t m = taps - 1u; m > 0; m--) v += a.w.conv[(size_t)(taps - 1u - m) * C + ch] * (pos >= m ? a.ring[(size_t)((pos - m) % taps) * C + ch] : 0.0f);
    }
    return siluf(v + a.w.conv[(size_t)(taps - 1u) * C + ch] * now + a.w.conv_bias[ch]);
}

// One workgroup of 256 threads: (head, 16 rows of its state).  bc: LDS, B [np] | C [np] | x [kRows].  B and C are convolved by every workgroup of their group; one of them writes the newest inputs
// to the ring, into a slot nobody reads.
__device__ __forceinline__ void ssd_step_block(const SsdStepArgs& a, uint32_t block, float* bc) {
    const SsdShape& s = a.s;
    const uint32_t parts = s.pp / kRows, h = block / parts, part = block % parts, per = s.heads / s.groups, grp = h / per;
    const uint32_t tid = threadIdx.x, l16 = tid & 15u, p = part * kRows + (tid >> 4), C = s.channels(), np = s.np;
    const uint32_t xs = s.heads * s.pp, gn = s.groups * np;
    float* S = a.state + ((size_t)h * s.pp + p) * np;
    // requested before the convolution whose results they meet
    constexpr int AHEAD = 2;
    v4f st[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; i++) {
        const uint32_t e = 4u * l16 + 64u * i;
        st[i] = *reinterpret_cast<const v4f*>(S + (e < np ? e : 0u));
    }
    const uint32_t pos = *a.d_pos;
    const float dt_raw = a.p.p[a.p.dt_at + h], dt_bias = a.w.dt_bias[h], rate = a.w.rate[h], dskip = a.w.d[h], z = a.p.p[a.p.z_at + h * s.pp + p];
    for (uint32_t i = tid; i < 2u * np + kRows; i += 256) {
        const bool is_x = i >= 2u * np;
        const uint32_t ch = is_x ? h * s.pp + part * kRows + (i - 2u * np) : xs + (i < np ? 0u : gn) + grp * np + (i < np ? i : i - np);
        const float now = a.p.p[a.p.x_at + ch];
        bc[i] = conv_now(a, ch, pos, now);
        if (is_x || (part == 0 && h % per == 0)) a.ring[(size_t)(pos % s.taps) * C + ch] = now;
    }
    const float dt = softplusf(dt_raw + dt_bias), decay = pos == 0 ? 0.0f : expf(rate * dt);
    __syncthreads();
    const float x = bc[2u * np + (tid >> 4)], gain = dt * x;
    float y = 0.0f;
    auto piece = [&](uint32_t e, v4f v) {
        const v4f b = *reinterpret_cast<const v4f*>(bc + e), c = *reinterpret_cast<const v4f*>(bc + np + e);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            v[i] = pos == 0 ? gain * b[i] : decay * v[i] + gain * b[i];
            y += c[i] * v[i];
        }
        *reinterpret_cast<v4f*>(S + e) = v;
    };
#pragma unroll
    for (int i = 0; i < AHEAD; i++)
        if (4u * l16 + 64u * i < np) piece(4u * l16 + 64u * i, st[i]);
    for (uint32_t e = 4u * l16 + 64u * AHEAD; e < np; e += 64u) piece(e, *reinterpret_cast<const v4f*>(S + e));
    y = group_sum<16>(y);
    if (l16 == 0 && p < s.vdim) a.out[h * s.vdim + p] = (y + dskip * x) * siluf(z);
}

inline bool ssd_shape_ok(const SsdShape& s, const SsdProj& p) {
    return s.heads > 0 && s.groups > 0 && s.heads % s.groups == 0 && s.state > 0 && s.np >= s.state && s.np >= 32u && (s.np & (s.np - 1u)) == 0 &&
           s.np <= kSsdMaxState && s.pp >= s.vdim && s.pp % 16u == 0 && s.vdim > 0 && s.taps > 0 && s.taps <= kConvTokens && p.p &&
           (p.ldp | p.z_at | p.x_at) % 4u == 0;
}
inline uint32_t ssd_step_blocks(const SsdShape& s) { return s.heads * (s.pp / kRows); }
inline uint32_t ssd_step_lds(const SsdShape& s) { return (2u * s.np + kRows) * 4u; }

}  // namespace

}  // namespace wick_rocm
