// State-space duality: per head a matrix state with one decay, S_t = exp(rate dt_t) S_(t-1) + dt_t x_t B_t^T, read by C_t, behind a short
// convolution, with a gate on the result.  The state is f32, [vdim][state] per head, and so is everything that enters the recurrence.
//
//   step    one token: convolution, state, gate in one launch;
//   scan    a portion token by token, the state in registers, all arithmetic f32 (short portions, the f32 model);
//   chunks  64 tokens at a time on the matrix cores: every chunk's own contribution to the state, the states in front of the chunks, then a
//           chunk's outputs from the tokens before it in the chunk (C B^T, masked and weighted, times x) and from the state in front of it.
//           x, B and C are bfloat16; weights, decays and states, f32 quantities, enter the products as two bfloat16 terms.
#include "ssd_step.h"

namespace wick_rocm {

namespace {

typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));

constexpr uint32_t kChunk = 64;
__global__ __launch_bounds__(256) void ssd_step_kernel(SsdStepArgs a) {
    extern __shared__ __align__(16) float bc[];
    ssd_step_block(a, blockIdx.x, bc);
}

// ---- token by token -----------------------------------------------------------------------------------------------------------
// The convolution's results as f32 rows.
struct ConvToRows {
    float* u;
    uint32_t channels;
    __device__ void operator()(uint32_t ch, uint32_t t0, const float (&v)[kConvTokens], uint32_t count) const {
#pragma unroll
        for (uint32_t i = 0; i < kConvTokens; i++)
            if (i < count) u[(size_t)(t0 + i) * channels + ch] = siluf(v[i]);
    }
};

struct ScanArgs {
    SsdShape s;
    SsdWeights w;
    SsdProj p;
    const float* u;
    float *state, *out;
    uint32_t n, pos0, ldo;
};

// Workgroup (head, 16 rows of its state); the next token's operands are in flight during this one's.
template <int NI>
__global__ __launch_bounds__(256) void ssd_scan_kernel(ScanArgs a) {
    const SsdShape& s = a.s;
    const uint32_t parts = s.pp / kRows, h = blockIdx.x / parts, part = blockIdx.x % parts, grp = h / (s.heads / s.groups);
    const uint32_t tid = threadIdx.x, l16 = tid & 15u, p = part * kRows + (tid >> 4), C = s.channels(), np = s.np;
    const uint32_t b_at = s.heads * s.pp + grp * np, c_at = b_at + s.groups * np;
    float* S = a.state + ((size_t)h * s.pp + p) * np;
    const float bias = a.w.dt_bias[h], rate = a.w.rate[h], dskip = a.w.d[h];
    v4f st[NI];
#pragma unroll
    for (int i = 0; i < NI; i++) {
        const uint32_t e = 4u * l16 + 64u * i;
        st[i] = a.pos0 > 0 && e < np ? *reinterpret_cast<const v4f*>(S + e) : v4f{0.f, 0.f, 0.f, 0.f};
    }
    struct Token {
        v4f b[NI], c[NI];
        float x, dt, z;
    } tok[2];
    auto load = [&](Token& k, uint32_t t) {
        const float* u = a.u + (size_t)t * C;
        const float* q = a.p.p + (size_t)t * a.p.ldp;
#pragma unroll
        for (int i = 0; i < NI; i++) {
            const uint32_t e = 4u * l16 + 64u * i < np ? 4u * l16 + 64u * i : 0u;
            k.b[i] = *reinterpret_cast<const v4f*>(u + b_at + e), k.c[i] = *reinterpret_cast<const v4f*>(u + c_at + e);
        }
        k.x = u[h * s.pp + p], k.dt = q[a.p.dt_at + h], k.z = q[a.p.z_at + h * s.pp + p];
    };
    auto step = [&](const Token& k, uint32_t t) {
        const float dt = softplusf(k.dt + bias), decay = expf(rate * dt), gain = dt * k.x;
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < NI; i++) {
            if (4u * l16 + 64u * i >= np) continue;
#pragma unroll
            for (int j = 0; j < 4; j++) st[i][j] = decay * st[i][j] + gain * k.b[i][j], y += k.c[i][j] * st[i][j];
        }
        y = group_sum<16>(y);
        if (l16 == 0 && p < s.vdim) a.out[(size_t)t * a.ldo + h * s.vdim + p] = (y + dskip * k.x) * siluf(k.z);
    };
    load(tok[0], 0);
    for (uint32_t t = 0; t < a.n; t += 2) {
        load(tok[1], t + 1u < a.n ? t + 1u : t);
        step(tok[0], t);
        if (t + 1u >= a.n) break;
        load(tok[0], t + 2u < a.n ? t + 2u : t);
        step(tok[1], t + 1u);
    }
#pragma unroll
    for (int i = 0; i < NI; i++)
        if (4u * l16 + 64u * i < np) *reinterpret_cast<v4f*>(S + 4u * l16 + 64u * i) = st[i];
}

// ---- chunks -------------------------------------------------------------------------------------------------------------------
// x and B channel by channel in tiles of 64 tokens (zeros behind the portion), B and C token by token.
struct ConvToTiles {
    uint16_t *tiles, *rows;
    uint32_t xs, gn;  // channels of x, of B (and of C)
    __device__ void operator()(uint32_t ch, uint32_t t0, const float (&v)[kConvTokens], uint32_t count) const {
        bf8 b;
#pragma unroll
        for (uint32_t i = 0; i < kConvTokens; i++) b[i] = i < count ? (__bf16)(v[i] * sigmoid_hw(v[i])) : (__bf16)0.0f;
        if (ch < xs + gn) *reinterpret_cast<bf8*>(tiles + ((size_t)(t0 / kChunk) * (xs + gn) + ch) * kChunk + t0 % kChunk) = b;
        if (ch >= xs) {
#pragma unroll
            for (uint32_t i = 0; i < kConvTokens; i++) {
                const __bf16 one = b[i];
                rows[(size_t)(t0 + i) * 2u * gn + ch - xs] = __builtin_bit_cast(uint16_t, one);
            }
        }
    }
};

struct ChunkArgs {
    SsdShape s;
    SsdWeights w;
    SsdProj p;
    SsdScratch k;
    float *state, *out;
    uint32_t n, pos0, chunks, ldo;
    __device__ float* meta(uint32_t c, uint32_t h) const { return k.meta + ((size_t)c * s.heads + h) * 2u * kChunk; }     // [cumulated log decay | dt]
    __device__ float* total(uint32_t c, uint32_t h) const { return k.meta + (size_t)chunks * s.heads * 2u * kChunk + (size_t)c * s.heads + h; }
    __device__ const uint16_t* tile(uint32_t c, uint32_t ch) const { return k.tiles + ((size_t)c * (s.heads * s.pp + s.groups * s.np) + ch) * kChunk; }
};

__device__ __forceinline__ void split_terms(float v, __bf16& hi, __bf16& lo) {
    hi = (__bf16)v;
    lo = (__bf16)(v - (float)hi);
}

// Workgroup (chunk, head): the chunk's steps and decays, and its own contribution to the state, x (w B)^T with w_j the step of token j
// and its decay to the chunk's end.
__global__ __launch_bounds__(256) void ssd_sums_kernel(ChunkArgs a) {
    __shared__ __align__(16) float wt[kChunk];
    const SsdShape& s = a.s;
    const uint32_t c = blockIdx.x, h = blockIdx.y, grp = h / (s.heads / s.groups);
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4;
    if (wave == 0) {
        const uint32_t t = c * kChunk + lane;
        const float dt = t < a.n ? softplusf(a.p.p[(size_t)t * a.p.ldp + a.p.dt_at + h] + a.w.dt_bias[h]) : 0.0f;
        float cum = a.w.rate[h] * dt;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const float o = __shfl_up(cum, d, 64);
            if (lane >= (uint32_t)d) cum += o;
        }
        const float total = __shfl(cum, 63, 64);
        wt[lane] = expf(total - cum) * dt;
        float* m = a.meta(c, h);
        m[lane] = cum, m[kChunk + lane] = dt;
        if (lane == 0) *a.total(c, h) = expf(total);
    }
    __syncthreads();
    const uint16_t* xt = a.tile(c, h * s.pp);
    const uint16_t* bt = a.tile(c, s.heads * s.pp + grp * s.np);
    float* out = a.k.sums + ((size_t)c * s.heads + h) * s.pp * s.np;
    for (uint32_t nt = wave; nt < s.np / 16u; nt += 4u) {
        bf8 bh[2], bl[2];
#pragma unroll
        for (int k = 0; k < 2; k++) {
            const bf8 b = *reinterpret_cast<const bf8*>(bt + (size_t)(16u * nt + l16) * kChunk + 32u * k + 8u * g);
            const v4f w0 = *reinterpret_cast<const v4f*>(&wt[32 * k + 8 * g]), w1 = *reinterpret_cast<const v4f*>(&wt[32 * k + 8 * g + 4]);
#pragma unroll
            for (int j = 0; j < 8; j++) {
                __bf16 hi, lo;
                split_terms((float)b[j] * (j < 4 ? w0[j & 3] : w1[j & 3]), hi, lo);
                bh[k][j] = hi, bl[k][j] = lo;
            }
        }
        for (uint32_t pt = 0; pt < s.pp / 16u; pt++) {
            v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 2; k++) {
                const bf8 x = *reinterpret_cast<const bf8*>(xt + (size_t)(16u * pt + l16) * kChunk + 32u * k + 8u * g);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, bl[k], acc, 0, 0, 0);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, bh[k], acc, 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < 4; r++) out[(size_t)(16u * pt + 4u * g + r) * s.np + 16u * nt + l16] = acc[r];
        }
    }
}

// The states in front of the chunks, four elements a thread.
__global__ __launch_bounds__(256) void ssd_starts_kernel(ChunkArgs a) {
    const SsdShape& s = a.s;
    const uint32_t each = s.pp * s.np, all = s.heads * each, e = 4u * (blockIdx.x * 256u + threadIdx.x);
    if (e >= all) return;
    const uint32_t h = e / each, in = e % each;
    v4f S = a.pos0 > 0 ? *reinterpret_cast<const v4f*>(a.state + e) : v4f{0.f, 0.f, 0.f, 0.f};
    constexpr uint32_t B = 8;
    for (uint32_t c0 = 0; c0 < a.chunks; c0 += B) {
        v4f add[B];
        float dec[B];
#pragma unroll
        for (uint32_t i = 0; i < B; i++) {
            const uint32_t c = c0 + i < a.chunks ? c0 + i : a.chunks - 1u;
            add[i] = *reinterpret_cast<const v4f*>(a.k.sums + (size_t)c * all + e), dec[i] = *a.total(c, h);
        }
#pragma unroll
        for (uint32_t i = 0; i < B; i++) {
            if (c0 + i >= a.chunks) break;
            bf4 hi, lo;
#pragma unroll
            for (int j = 0; j < 4; j++) {
                __bf16 u, v;
                split_terms(S[j], u, v);
                hi[j] = u, lo[j] = v;
            }
            uint16_t* o = a.k.starts + ((size_t)(c0 + i) * s.heads + h) * 2u * each + in;
            *reinterpret_cast<bf4*>(o) = hi, *reinterpret_cast<bf4*>(o + each) = lo;
            S = S * dec[i] + add[i];
        }
    }
    *reinterpret_cast<v4f*>(a.state + e) = S;
}

// Workgroup (chunk, head), 16 tokens per wave.  Scores transposed, S^T[j][i] = B_j . C_i, so that the weighted scores go into the second
// product in the registers they are in: slot k of lane group g stands for token 4 g + k of a 16-token sub-tile (k < 4) or of the
// next one (k >= 4) in both operands.  Results transposed, Y^T[p][i]: a lane holds four neighbouring coordinates of one token.
template <int NK>
__global__ __launch_bounds__(256) void ssd_outputs_kernel(ChunkArgs a) {
    const SsdShape& s = a.s;
    const uint32_t c = blockIdx.x, h = blockIdx.y, grp = h / (s.heads / s.groups), gn = s.groups * s.np;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4;
    const uint32_t i = 16u * wave + l16, t = c * kChunk + i;
    if (c * kChunk + 16u * wave >= a.n) return;
    const uint16_t* rows = a.k.rows + (size_t)c * kChunk * 2u * gn + grp * s.np;
    bf8 cf[NK];
#pragma unroll
    for (int k = 0; k < NK; k++) cf[k] = *reinterpret_cast<const bf8*>(rows + (size_t)i * 2u * gn + gn + 32u * k + 8u * g);
    const float* m = a.meta(c, h);
    const float cum_i = m[i];
    bf8 ph[2], pl[2];
#pragma unroll
    for (int u = 0; u < 4; u++) {
        v4f sc = {0.f, 0.f, 0.f, 0.f};
        if ((uint32_t)u <= wave) {
#pragma unroll
            for (int k = 0; k < NK; k++) {
                const bf8 b = *reinterpret_cast<const bf8*>(rows + (size_t)(16u * u + l16) * 2u * gn + 32u * k + 8u * g);
                sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, cf[k], sc, 0, 0, 0);
            }
        }
        const v4f cum_j = *reinterpret_cast<const v4f*>(m + 16 * u + 4 * g), dt_j = *reinterpret_cast<const v4f*>(m + kChunk + 16 * u + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float w = 16u * u + 4u * g + r <= i ? sc[r] * expf(cum_i - cum_j[r]) * dt_j[r] : 0.0f;
            __bf16 hi, lo;
            split_terms(w, hi, lo);
            ph[u >> 1][4 * (u & 1) + r] = hi, pl[u >> 1][4 * (u & 1) + r] = lo;
        }
    }
    const float past = expf(cum_i), dskip = a.w.d[h];
    const uint32_t each = s.pp * s.np;
    const uint16_t* start = a.k.starts + ((size_t)c * s.heads + h) * 2u * each;
    for (uint32_t pt = 0; pt < s.pp / 16u; pt++) {
        const uint16_t* xr = a.tile(c, h * s.pp + 16u * pt + l16);
        v4f o = {0.f, 0.f, 0.f, 0.f}, q = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < NK; k++) {
            const uint16_t* sr = start + (size_t)(16u * pt + l16) * s.np + 32u * k + 8u * g;
            q = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf8*>(sr + each), cf[k], q, 0, 0, 0);
            q = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf8*>(sr), cf[k], q, 0, 0, 0);
        }
#pragma unroll
        for (int u = 0; u < 2; u++) {
            if (2u * u > wave) continue;
            const bf4 v0 = *reinterpret_cast<const bf4*>(xr + 32 * u + 4 * g), v1 = *reinterpret_cast<const bf4*>(xr + 32 * u + 16 + 4 * g);
            const bf8 v = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
            o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl[u], o, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph[u], o, 0, 0, 0);
        }
        if (t >= a.n) continue;
        const uint32_t p = 16u * pt + 4u * g;
        const v4f z = *reinterpret_cast<const v4f*>(a.p.p + (size_t)t * a.p.ldp + a.p.z_at + h * s.pp + p);
        float* out = a.out + (size_t)t * a.ldo + h * s.vdim + p;
        v4f y;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float x = __uint_as_float((uint32_t)a.tile(c, h * s.pp + p + r)[i] << 16);
            y[r] = (o[r] + past * q[r] + dskip * x) * (z[r] * sigmoid_hw(z[r]));
        }
        if (s.vdim % 4u == 0) {
            if (p < s.vdim) *reinterpret_cast<v4f*>(out) = y;
        } else {
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (p + r < s.vdim) out[r] = y[r];
        }
    }
}

ShortConv conv_of(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, uint32_t pos0) {
    return ShortConv{p.p + p.x_at, p.ldp, s.channels(), s.taps, pos0, w.conv, w.conv_bias, ring};
}

}  // namespace

hipError_t launch_ssd_step(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, float* out, const uint32_t* d_pos, const Launch& L) {
    if (!ssd_shape_ok(s, p) || !d_pos) return hipErrorInvalidValue;
    return launch_kernel_lds(L, kFamOther, ssd_step_kernel, dim3(ssd_step_blocks(s)), dim3(256), ssd_step_lds(s),
                             SsdStepArgs{s, w, p, ring, state, out, d_pos});
}

hipError_t launch_ssd_scan(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, float* rows, uint32_t n, uint32_t pos0,
                           float* out, uint32_t ldo, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!ssd_shape_ok(s, p) || ldo < s.heads * s.vdim) return hipErrorInvalidValue;
    const hipError_t e = launch_short_conv(conv_of(s, w, p, ring, pos0), n, n, ConvToRows{rows, s.channels()}, L);
    if (e != hipSuccess) return e;
    const ScanArgs a{s, w, p, rows, state, out, n, pos0, ldo};
    const dim3 grid(s.heads * (s.pp / kRows));
    if (s.np <= 64u) return launch_kernel(L, kFamOther, ssd_scan_kernel<1>, grid, dim3(256), a);
    if (s.np <= 128u) return launch_kernel(L, kFamOther, ssd_scan_kernel<2>, grid, dim3(256), a);
    if (s.np <= 256u) return launch_kernel(L, kFamOther, ssd_scan_kernel<4>, grid, dim3(256), a);
    return launch_kernel(L, kFamOther, ssd_scan_kernel<8>, grid, dim3(256), a);
}

hipError_t launch_ssd_chunks(const SsdShape& s, const SsdWeights& w, const SsdProj& p, float* ring, float* state, const SsdScratch& scratch, uint32_t n,
                             uint32_t pos0, float* out, uint32_t ldo, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!ssd_shape_ok(s, p) || ldo < s.heads * s.vdim || ldo % 4u) return hipErrorInvalidValue;
    const uint32_t chunks = ssd_chunks(n), xs = s.heads * s.pp, gn = s.groups * s.np;
    hipError_t e = launch_short_conv(conv_of(s, w, p, ring, pos0), n, chunks * kChunk, ConvToTiles{scratch.tiles, scratch.rows, xs, gn}, L);
    if (e != hipSuccess) return e;
    const ChunkArgs a{s, w, p, scratch, state, out, n, pos0, chunks, ldo};
    const dim3 grid(chunks, s.heads);
    if ((e = launch_kernel(L, kFamOther, ssd_sums_kernel, grid, dim3(256), a)) != hipSuccess) return e;
    if ((e = launch_kernel(L, kFamOther, ssd_starts_kernel, dim3((s.heads * s.pp * s.np / 4u + 255u) / 256u), dim3(256), a)) != hipSuccess) return e;
    switch (s.np) {
        case 32: return launch_kernel(L, kFamOther, ssd_outputs_kernel<1>, grid, dim3(256), a);
        case 64: return launch_kernel(L, kFamOther, ssd_outputs_kernel<2>, grid, dim3(256), a);
        case 128: return launch_kernel(L, kFamOther, ssd_outputs_kernel<4>, grid, dim3(256), a);
        case 256: return launch_kernel(L, kFamOther, ssd_outputs_kernel<8>, grid, dim3(256), a);
        case 512: return launch_kernel(L, kFamOther, ssd_outputs_kernel<16>, grid, dim3(256), a);
        default: return hipErrorInvalidValue;
    }
}

}  // namespace wick_rocm
