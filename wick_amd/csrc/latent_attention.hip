// Attention over a cached latent: every position keeps one row, the normed latent c and the rotated key part that all heads share.
// A head's key is [W_uk c | rotated part] and its value W_uv c, so a query can be taken either way:
//   absorbed   q . (W_uk c) = (W_uk^T q) . c: the query moves into the latent's space once and the cache rows serve as keys and as
//              values of all heads (the value expansion is applied to the weighted sum).  All arithmetic f32.  Decode steps, short
//              portions and the f32 model.
//   expanded   keys and values of all positions are made by two products and a prompt's queries walk them on the matrix cores:
//              fewer multiplications per (query, key) pair when there are many queries.
// Softmax is streamed over tiles of 64 positions in f32; position i sees every j <= i.
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));
typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
typedef uint32_t u4 __attribute__((ext_vector_type(4)));

constexpr uint32_t kChunk = 64;      // positions per pass
constexpr uint32_t kMaxSplits = 64;  // workgroups along the sequence
constexpr uint32_t kSlab = 128;      // latent columns per workgroup of the absorbing launch
constexpr uint32_t kStageBytes = 136u * 1024u;  // dynamic LDS of the staged form, beside at most 21 KB of its own
constexpr float kLog2e = 1.44269504088896340736f;

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(uint16_t* p, float v) { *p = __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ float widen_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float widen_hi(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }

// Pairs (2i, 2i + 1) of v turned by the position's angle of pair i.
__device__ __forceinline__ void rotate_pair(const float* rope, uint32_t pos, uint32_t half, uint32_t i, float& u, float& v) {
    const float c = rope[((size_t)pos * half + i) * 2], s = rope[((size_t)pos * half + i) * 2 + 1], u0 = u;
    u = u0 * c - v * s, v = v * c + u0 * s;
}

// The cache row of one position by a workgroup of 256 threads: d = [latent before its norm | key part before its rotation].
template <typename CT>
__device__ __forceinline__ void write_cache_row(const LatentShape& s, const LatentWeights& w, const float* d, uint32_t pos, CT* row) {
    __shared__ float slots[4];
    float ss = 0.0f;
    for (uint32_t e = threadIdx.x; e < s.rank; e += 256) ss += d[e] * d[e];
    ss = wave_sum_f32(ss);
    if ((threadIdx.x & 63u) == 0) slots[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf(((slots[0] + slots[1]) + (slots[2] + slots[3])) / (float)s.rank + s.eps);
    for (uint32_t e = threadIdx.x; e < s.rank_p; e += 256) put(row + e, e < s.rank ? d[e] * inv * w.norm[e] : 0.0f);
    const uint32_t half = s.rot / 2u;
    for (uint32_t i = threadIdx.x; i < s.rot_p / 2u; i += 256) {
        float u = 0.0f, v = 0.0f;
        if (i < half) {
            u = d[s.rank + 2 * i], v = d[s.rank + 2 * i + 1];
            rotate_pair(w.rope, pos, half, i, u, v);
        }
        put(row + s.rank_p + 2 * i, u), put(row + s.rank_p + 2 * i + 1, v);
    }
}

struct AbsorbArgs {
    LatentShape s;
    LatentWeights w;
    const float* proj;
    uint32_t ldp, pos0;
    const uint32_t* d_pos;
    void* cache;
    float* qa;
};

// Workgroups (head, slab of latent columns) absorb the queries of token blockIdx.y; the last one writes the token's cache row.
template <typename CT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(AbsorbArgs a) {
    __shared__ __align__(16) float red[8][kSlab];
    const LatentShape& s = a.s;
    const uint32_t t = blockIdx.y, pos = (a.d_pos ? *a.d_pos : a.pos0) + t, tid = threadIdx.x;
    const uint32_t slabs = (s.rank_p + kSlab - 1u) / kSlab, qd = s.dim + s.rot;
    if (pos >= s.max_seq) return;  // the host checks by-value positions; a device-side one past the cache is dropped
    const float* p = a.proj + (size_t)t * a.ldp;
    if (blockIdx.x == s.heads * slabs) {
        write_cache_row(s, a.w, p + (size_t)s.heads * qd, pos, static_cast<CT*>(a.cache) + (size_t)pos * s.row());
        return;
    }
    const uint32_t h = blockIdx.x / slabs, slab = blockIdx.x % slabs;
    const float* q = p + (size_t)h * qd;
    float* out = a.qa + ((size_t)t * s.heads + h) * s.row();
    const uint32_t grp = tid >> 5, col = slab * kSlab + 4u * (tid & 31u);
    v4f acc = {0.f, 0.f, 0.f, 0.f};
    if (col < s.rank_p) {
        const uint16_t* w = a.w.uk + (size_t)h * s.dim * s.rank_p + col;
#pragma unroll 8
        for (uint32_t d = grp; d < s.dim; d += 8) {
            const uint2 k = *reinterpret_cast<const uint2*>(w + (size_t)d * s.rank_p);
            const float qv = q[d];
            acc[0] = fmaf(qv, widen_lo(k.x), acc[0]), acc[1] = fmaf(qv, widen_hi(k.x), acc[1]);
            acc[2] = fmaf(qv, widen_lo(k.y), acc[2]), acc[3] = fmaf(qv, widen_hi(k.y), acc[3]);
        }
    }
    *reinterpret_cast<v4f*>(&red[grp][4u * (tid & 31u)]) = acc;
    __syncthreads();
    if (tid < kSlab && slab * kSlab + tid < s.rank_p) {
        float v = 0.0f;
#pragma unroll
        for (int g = 0; g < 8; g++) v += red[g][tid];
        out[slab * kSlab + tid] = v;
    }
    if (slab == 0) {
        const uint32_t half = s.rot / 2u;
        for (uint32_t i = tid; i < s.rot_p / 2u; i += 256) {
            float u = 0.0f, v = 0.0f;
            if (i < half) {
                u = q[s.dim + 2 * i], v = q[s.dim + 2 * i + 1];
                rotate_pair(a.w.rope, pos, half, i, u, v);
            }
            out[s.rank_p + 2 * i] = u, out[s.rank_p + 2 * i + 1] = v;
        }
    }
}

// One workgroup per token: its cache row, and every head's query with its rotated part turned, as bfloat16 hi | lo.
__global__ __launch_bounds__(256) void latent_rope_kernel(AbsorbArgs a, uint16_t* __restrict__ qout, uint32_t dqp) {
    const LatentShape& s = a.s;
    const uint32_t t = blockIdx.x, pos = a.pos0 + t, qd = s.dim + s.rot, half = s.rot / 2u;
    if (pos >= s.max_seq) return;
    const float* p = a.proj + (size_t)t * a.ldp;
    write_cache_row(s, a.w, p + (size_t)s.heads * qd, pos, static_cast<uint16_t*>(a.cache) + (size_t)pos * s.row());
    for (uint32_t i = threadIdx.x; i < s.heads * dqp; i += 256) {
        const uint32_t h = i / dqp, e = i % dqp;
        float v = 0.0f;
        if (e < s.dim) {
            v = p[h * qd + e];
        } else if (e < qd) {
            const uint32_t k = (e - s.dim) >> 1;
            float u = p[h * qd + s.dim + 2 * k], w = p[h * qd + s.dim + 2 * k + 1];
            rotate_pair(a.w.rope, pos, half, k, u, w);
            v = (e - s.dim) & 1u ? w : u;
        }
        const float hi = (float)(__bf16)v;
        uint16_t* o = qout + ((size_t)t * s.heads + h) * 2u * dqp + e;
        put(o, hi), put(o + dqp, v - hi);
    }
}

// ---- absorbed attention ----------------------------------------------------------------------------------------------------
struct AttendArgs {
    LatentShape s;
    const float* qa;
    const void* cache;
    float* part;          // [n][heads][splits][rank_p + 4]: {max, sum, -, -, weighted latents}
    uint32_t pos0, splits;
    const uint32_t* d_pos;
};

template <typename CT>
__device__ __forceinline__ void load8(const CT* p, float (&v)[8]) {
    if constexpr (sizeof(CT) == 2) {
        const uint4 w = *reinterpret_cast<const uint4*>(p);
        v[0] = widen_lo(w.x), v[1] = widen_hi(w.x), v[2] = widen_lo(w.y), v[3] = widen_hi(w.y);
        v[4] = widen_lo(w.z), v[5] = widen_hi(w.z), v[6] = widen_lo(w.w), v[7] = widen_hi(w.w);
    } else {
        const v4f a = *reinterpret_cast<const v4f*>(p), b = *reinterpret_cast<const v4f*>(p + 4);
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] = a[i], v[4 + i] = b[i];
    }
}

// Workgroup (split, HG heads, token).  STAGED: a chunk's cache rows are brought into LDS once (all of a thread's loads in flight
// together) and serve both halves; rows too long for that are read from memory twice.  Scores: 16 lanes walk the pieces of four
// cache rows at a time, so a piece of a query is read from LDS once for four positions.  Values: a thread owns NP pairs of latent
// columns for all HG heads.
template <int HG, int NP, bool STAGED, typename CT>
__global__ __launch_bounds__(256) void latent_attend_kernel(AttendArgs a) {
    extern __shared__ __align__(16) float qs[];  // [HG][row], then STAGED: [kChunk][row] of the cache type
    __shared__ __align__(16) float sc[HG][kChunk], wt[kChunk][HG];
    __shared__ float corr[HG];
    __shared__ float2 red[HG][256];
    const LatentShape& s = a.s;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, row = s.row();
    const uint32_t split = blockIdx.x, h0 = blockIdx.y * HG, t = blockIdx.z;
    const uint32_t nh = s.heads - h0 < (uint32_t)HG ? s.heads - h0 : (uint32_t)HG;
    const float* qa = a.qa + ((size_t)t * s.heads + h0) * row;  // rows of a token's heads follow each other
    const uint32_t q_len = nh * row;
    const v4f q_first = 4u * tid < q_len ? *reinterpret_cast<const v4f*>(qa + 4u * tid) : v4f{0.f, 0.f, 0.f, 0.f};
    const uint32_t pos = (a.d_pos ? *a.d_pos : a.pos0) + t;
    if (pos >= s.max_seq || split * kChunk > pos) return;  // the merge derives the number of partials from pos as well
    const CT* cache = static_cast<const CT*>(a.cache);
    constexpr uint32_t PER = 16 / sizeof(CT), AHEAD = 12;  // elements of a 16-byte piece; pieces a thread has in flight
    u4 ahead[STAGED ? AHEAD : 1];
    auto fetch = [&](const CT* rows, uint32_t pieces, uint32_t i0) {
#pragma unroll
        for (uint32_t j = 0; j < (STAGED ? AHEAD : 1u); j++) ahead[j] = *reinterpret_cast<const u4*>(rows + (size_t)(i0 + 256u * j < pieces ? i0 + 256u * j : 0u) * PER);
    };
    auto chunk_keys = [&](uint32_t c) { return pos + 1u - c * kChunk < kChunk ? pos + 1u - c * kChunk : kChunk; };
    if constexpr (STAGED) fetch(cache + (size_t)split * kChunk * row, chunk_keys(split) * (row / PER), tid);  // ... before the queries
    for (uint32_t i = 4u * tid; i < HG * row; i += 1024u) {  // absent heads: zeros
        const v4f q = i == 4u * tid ? q_first : i < q_len ? *reinterpret_cast<const v4f*>(qa + i) : v4f{0.f, 0.f, 0.f, 0.f};
        *reinterpret_cast<v4f*>(qs + i) = q;
    }
    __syncthreads();
    const uint32_t pairs = s.rank_p / 2u;
    uint32_t cpp = 16;  // threads along the column pairs: a power of two
    while (cpp < 256u && cpp < pairs) cpp <<= 1;
    const uint32_t kgroups = 256u / cpp, cp = tid % cpp, kg = tid / cpp;
    float acc[NP][HG][2], m_run[(HG + 3) / 4], l_run[(HG + 3) / 4];
#pragma unroll
    for (int i = 0; i < NP; i++)
#pragma unroll
        for (int h = 0; h < HG; h++) acc[i][h][0] = acc[i][h][1] = 0.0f;
#pragma unroll
    for (int i = 0; i < (HG + 3) / 4; i++) m_run[i] = -__builtin_inff(), l_run[i] = 0.0f;
    const uint32_t l16 = lane & 15u, key_in = wave * 16u + (lane >> 4) * 4u;  // this lane group's four positions of a chunk

    for (uint32_t c = split; c * kChunk <= pos; c += a.splits) {
        const uint32_t t0 = c * kChunk, nt = chunk_keys(c);
        const CT* rows = cache + (size_t)t0 * row;
        if constexpr (STAGED) {
            CT* stage = reinterpret_cast<CT*>(qs + HG * row);
            const uint32_t pieces = nt * (row / PER);
            for (uint32_t i0 = tid; i0 < pieces; i0 += AHEAD * 256u) {
                if (c != split || i0 != tid) fetch(rows, pieces, i0);
#pragma unroll
                for (uint32_t j = 0; j < AHEAD; j++)
                    if (i0 + 256u * j < pieces) *reinterpret_cast<u4*>(stage + (size_t)(i0 + 256u * j) * PER) = ahead[j];
            }
            rows = stage;
            __syncthreads();
        }
        const CT* kr[4];
#pragma unroll
        for (int k = 0; k < 4; k++) kr[k] = rows + (size_t)(key_in + k < nt ? key_in + k : nt - 1u) * row;
        float dot[4][HG];
#pragma unroll
        for (int k = 0; k < 4; k++)
#pragma unroll
            for (int h = 0; h < HG; h++) dot[k][h] = 0.0f;
        for (uint32_t at = 8u * l16; at < row; at += 128u) {
            float kv[4][8];
#pragma unroll
            for (int k = 0; k < 4; k++) load8(kr[k] + at, kv[k]);
#pragma unroll
            for (int h = 0; h < HG; h++) {
                const v4f q0 = *reinterpret_cast<const v4f*>(qs + h * row + at), q1 = *reinterpret_cast<const v4f*>(qs + h * row + at + 4);
#pragma unroll
                for (int k = 0; k < 4; k++)
#pragma unroll
                    for (int i = 0; i < 4; i++) dot[k][h] = fmaf(q0[i], kv[k][i], fmaf(q1[i], kv[k][4 + i], dot[k][h]));
            }
        }
#pragma unroll
        for (int h = 0; h < HG; h++)
#pragma unroll
            for (int k = 0; k < 4; k++) {
                const float d = group_sum<16>(dot[k][h]);
                if (l16 == 0) sc[h][key_in + k] = key_in + k < nt ? d * s.scale : -__builtin_inff();
            }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < (HG + 3) / 4; i++) {
            const uint32_t h = wave + 4u * i;
            if (h < (uint32_t)HG) {
                const float v = sc[h][lane];
                const float m_new = fmaxf(m_run[i], wave_max_f32(v));  // a chunk has at least one visible position: finite
                const float e = lane < nt ? expf(v - m_new) : 0.0f;
                const float f = expf(m_run[i] - m_new);
                wt[lane][h] = e;
                l_run[i] = l_run[i] * f + wave_sum_f32(e);
                m_run[i] = m_new;
                if (lane == 0) corr[h] = f;
            }
        }
        __syncthreads();
#pragma unroll
        for (int h = 0; h < HG; h++) {
            const float f = corr[h];
#pragma unroll
            for (int i = 0; i < NP; i++) acc[i][h][0] *= f, acc[i][h][1] *= f;
        }
        if (cp < pairs) {
#pragma unroll 8
            for (uint32_t k = kg; k < nt; k += kgroups) {
                const CT* vr = rows + (size_t)k * row;
                float w[HG];
#pragma unroll
                for (int h = 0; h < HG; h++) w[h] = wt[k][h];
#pragma unroll
                for (int i = 0; i < NP; i++) {
                    const uint32_t p = cp + 256u * i;
                    if (i > 0 && p >= pairs) continue;
                    float v0, v1;
                    if constexpr (sizeof(CT) == 2) {
                        const uint32_t v = *reinterpret_cast<const uint32_t*>(vr + 2 * p);
                        v0 = widen_lo(v), v1 = widen_hi(v);
                    } else {
                        const float2 v = *reinterpret_cast<const float2*>(vr + 2 * p);
                        v0 = v.x, v1 = v.y;
                    }
#pragma unroll
                    for (int h = 0; h < HG; h++) acc[i][h][0] = fmaf(w[h], v0, acc[i][h][0]), acc[i][h][1] = fmaf(w[h], v1, acc[i][h][1]);
                }
            }
        }
        __syncthreads();  // sc, wt and corr are rewritten by the next chunk
    }
    auto part_of = [&](int h) { return a.part + (((size_t)t * s.heads + h0 + h) * a.splits + split) * (s.rank_p + 4u); };
#pragma unroll
    for (int h = 0; h < HG; h++)
        if (h < (int)nh && wave == (uint32_t)(h & 3) && lane == 0) part_of(h)[0] = m_run[h >> 2], part_of(h)[1] = l_run[h >> 2];
#pragma unroll
    for (int i = 0; i < NP; i++) {
        if (i > 0) __syncthreads();
#pragma unroll
        for (int h = 0; h < HG; h++) red[h][tid] = float2{acc[i][h][0], acc[i][h][1]};
        __syncthreads();
        for (uint32_t x = tid; x < HG * cpp; x += 256u) {
            const uint32_t h = x / cpp, p = x % cpp + 256u * i;
            if (h >= nh || p >= pairs) continue;
            float2 v = {0.0f, 0.0f};
            for (uint32_t g = 0; g < kgroups; g++) v.x += red[h][g * cpp + x % cpp].x, v.y += red[h][g * cpp + x % cpp].y;
            float* part = part_of((int)h) + 4 + 2 * p;
            part[0] = v.x, part[1] = v.y;
        }
    }
}

struct MergeArgs {
    LatentShape s;
    const float* part;
    uint32_t pos0, splits;
    const uint32_t* d_pos;
    const uint16_t* uv;
    void* out;
    uint32_t ldo, kp;
};

// Workgroup (head, token, share of the head's values): the partials of the head become one weighted latent in LDS, then W_uv of it.
template <typename OT>
__global__ __launch_bounds__(256) void latent_merge_kernel(MergeArgs a) {
    extern __shared__ __align__(16) float oc[];  // [rank_p]
    __shared__ float wts[kMaxSplits];
    __shared__ v4f sums[256];
    const LatentShape& s = a.s;
    const uint32_t h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, lane = tid & 63u;
    // the first four value rows of a wave are requested before the partials are looked at (rank_p <= 512: whole rows)
    const uint32_t waves = gridDim.z * 4u, first = blockIdx.z * 4u + (tid >> 6);
    float ahead[4][8];
#pragma unroll
    for (int r = 0; r < 4; r++) {
        const uint32_t v = first + r * waves < s.vdim ? first + r * waves : s.vdim - 1u;
        if (8u * lane < s.rank_p) load8(a.uv + ((size_t)h * s.vdim + v) * s.rank_p + 8u * lane, ahead[r]);
    }
    const uint32_t stride = s.rank_p + 4u;
    const float* parts = a.part + ((size_t)t * s.heads + h) * a.splits * stride;
    // thread (group of partials, four latent columns)
    const uint32_t quads = s.rank_p / 4u;
    uint32_t cols = 8;
    while (cols < 256u && cols < quads) cols <<= 1;
    const uint32_t groups = 256u / cols, grp = tid / cols;
    v4f pre[8];
    auto fetch = [&](uint32_t quad, uint32_t i0) {
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const uint32_t i = i0 + j * groups;
            pre[j] = quad < quads ? *reinterpret_cast<const v4f*>(parts + (size_t)(i < a.splits ? i : 0u) * stride + 4 + 4 * quad) : v4f{0.f, 0.f, 0.f, 0.f};
        }
    };
    fetch(tid % cols, grp);
    const float m_raw = parts[(size_t)(tid < a.splits ? tid : 0u) * stride], l_raw = parts[(size_t)(tid < a.splits ? tid : 0u) * stride + 1];
    const uint32_t pos = (a.d_pos ? *a.d_pos : a.pos0) + t;
    if (pos >= s.max_seq) return;
    uint32_t active = pos / kChunk + 1u;  // what lies behind the active partials is from earlier steps: loaded, not used
    active = active < a.splits ? active : a.splits;
    if (tid < 64) {
        const bool on = tid < active;
        const float m_i = on ? m_raw : -__builtin_inff(), l_i = on ? l_raw : 0.0f;
        const float m = wave_max_f32(m_i), w = on ? expf(m_i - m) : 0.0f, l = wave_sum_f32(l_i * w);
        wts[tid] = w / l;
    }
    __syncthreads();
    for (uint32_t quad = tid % cols; quad < quads || quad == tid % cols; quad += cols) {
        v4f v = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t i0 = grp; i0 < active; i0 += 8u * groups) {
            if (quad != tid % cols || i0 != grp) fetch(quad, i0);
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const uint32_t i = i0 + j * groups;
                if (i < active) v += pre[j] * wts[i];
            }
        }
        if (groups > 1) {  // then one quad per thread (cols >= quads)
            sums[tid] = v;
            __syncthreads();
            if (grp == 0) {
                v = sums[tid];
                for (uint32_t g = 1; g < groups; g++) v += sums[g * cols + tid];
            }
        }
        if (grp == 0 && quad < quads) *reinterpret_cast<v4f*>(oc + 4 * quad) = v;
    }
    __syncthreads();
    OT* out = static_cast<OT*>(a.out) + (size_t)t * a.ldo;
    for (uint32_t v0 = first; v0 < s.vdim; v0 += 4u * waves) {
        float d[4] = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t at = 8u * lane; at < s.rank_p; at += 512u) {
            const v4f o0 = *reinterpret_cast<const v4f*>(oc + at), o1 = *reinterpret_cast<const v4f*>(oc + at + 4);
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const uint32_t v = v0 + r * waves < s.vdim ? v0 + r * waves : v0;
                float w[8];
                if (v0 == first && at < 512u) {
#pragma unroll
                    for (int i = 0; i < 8; i++) w[i] = ahead[r][i];
                } else {
                    load8(a.uv + ((size_t)h * s.vdim + v) * s.rank_p + at, w);
                }
#pragma unroll
                for (int i = 0; i < 4; i++) d[r] = fmaf(w[i], o0[i], fmaf(w[4 + i], o1[i], d[r]));
            }
        }
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float o = wave_sum_f32(d[r]);
            if (lane == 0 && v0 + r * waves < s.vdim) put(out + h * s.vdim + v0 + r * waves, o);
        }
    }
    if (h + 1 == s.heads && blockIdx.z == 0)
        for (uint32_t e = s.heads * s.vdim + tid; e < a.kp; e += 256) put(out + e, 0.0f);
}

// ---- a prompt's queries over expanded keys and values --------------------------------------------------------------------------
struct PrefillArgs {
    const uint16_t *q, *kx, *vt;   // [n][heads][2][DQ], [keys][ldk] = [heads][DQ], [heads * DV][ldv]
    uint32_t ldk, ldv, n, pos0, heads, vdim;
    float scale_log2;
    uint16_t* out;
    uint32_t ldo, kp;
};

// Workgroup: one head, 64 queries, 16 per wave; 64 positions at a time through LDS, the next tile's loads in flight meanwhile.
//   scores transposed: S^T[key][query], A = K, B = Q^T (hi and lo term of the query): lane l holds keys 4 (l / 16) + r of query l % 16;
//   values transposed: O^T[d][query] += V^T[d][key] P[key][query], A = V^T, B = P: the weights go from one product into the next
//   in the registers they are in -- slot j of lane group g stands for key 4 g + j of a 16-key sub-tile (j < 4) or of the next one
//   (j >= 4) in both operands.  The weights enter as two bfloat16 terms, so they keep 16 bits.
template <int NS, int NV>
__global__ __launch_bounds__(256) void latent_prefill_kernel(PrefillArgs a) {
    constexpr uint32_t DQ = 32 * NS, DV = 16 * NV, LDK = DQ + 8, LDV = 72;
    __shared__ __align__(16) uint16_t ks[64 * LDK], vs[DV * LDV];
    const uint32_t h = blockIdx.x, qblocks = (a.n + 63u) / 64u, j0 = (qblocks - 1u - blockIdx.y) * 64u;  // the longest first
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4;
    const uint32_t jq = j0 + 16u * wave + l16, jl = jq < a.n ? jq : a.n - 1u, pq = a.pos0 + jl;
    const uint32_t wg_last = a.pos0 + (j0 + 63u < a.n ? j0 + 63u : a.n - 1u);
    const uint32_t wave_first = a.pos0 + j0 + 16u * wave, wave_last = wave_first + 15u < wg_last ? wave_first + 15u : wg_last;
    const bool active = j0 + 16u * wave < a.n;
    bf8 qh[NS], ql[NS];
    {
        const uint16_t* qp = a.q + ((size_t)jl * a.heads + h) * 2u * DQ + 8u * g;
#pragma unroll
        for (int i = 0; i < NS; i++) qh[i] = *reinterpret_cast<const bf8*>(qp + 32 * i), ql[i] = *reinterpret_cast<const bf8*>(qp + DQ + 32 * i);
    }
    v4f o[NV];
#pragma unroll
    for (int i = 0; i < NV; i++) o[i] = v4f{0.f, 0.f, 0.f, 0.f};
    float m_run = -__builtin_inff(), l_run = 0.0f;
    constexpr int KP = 64 * (DQ / 8) / 256, VP = DV * 8 / 256;
    u4 kr[KP], vr[VP];
    auto fetch = [&](uint32_t t0) {
#pragma unroll
        for (int i = 0; i < KP; i++) {
            const uint32_t c = tid + 256u * i, r = c / (DQ / 8), ch = c % (DQ / 8), key = t0 + r < wg_last ? t0 + r : wg_last;
            kr[i] = *reinterpret_cast<const u4*>(a.kx + (size_t)key * a.ldk + h * DQ + 8u * ch);
        }
#pragma unroll
        for (int i = 0; i < VP; i++) {
            const uint32_t c = tid + 256u * i, r = c >> 3, ch = c & 7u;
            vr[i] = *reinterpret_cast<const u4*>(a.vt + ((size_t)h * DV + r) * a.ldv + t0 + 8u * ch);
        }
    };
    fetch(0);
    for (uint32_t t0 = 0; t0 <= wg_last; t0 += 64u) {
        __syncthreads();  // the previous tile's reads are done
#pragma unroll
        for (int i = 0; i < KP; i++) {
            const uint32_t c = tid + 256u * i, r = c / (DQ / 8), ch = c % (DQ / 8);
            *reinterpret_cast<u4*>(&ks[r * LDK + 8u * ch]) = kr[i];
        }
#pragma unroll
        for (int i = 0; i < VP; i++) {
            const uint32_t c = tid + 256u * i, r = c >> 3, ch = c & 7u;
            *reinterpret_cast<u4*>(&vs[r * LDV + 8u * ch]) = vr[i];
        }
        __syncthreads();
        if (t0 + 64u <= wg_last) fetch(t0 + 64u);
        if (!active || t0 > wave_last) continue;
        v4f s[4];
#pragma unroll
        for (int u = 0; u < 4; u++) s[u] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NS; i++) {
            bf8 k[4];
#pragma unroll
            for (int u = 0; u < 4; u++) k[u] = *reinterpret_cast<const bf8*>(&ks[(16 * u + l16) * LDK + 32 * i + 8 * g]);
#pragma unroll
            for (int u = 0; u < 4; u++) s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[u], ql[i], s[u], 0, 0, 0);
#pragma unroll
            for (int u = 0; u < 4; u++) s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[u], qh[i], s[u], 0, 0, 0);
        }
        const bool masked = t0 + 63u > wave_first;
        float top = -__builtin_inff();
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                s[u][r] *= a.scale_log2;
                if (masked && t0 + 16u * u + 4u * g + r > pq) s[u][r] = -__builtin_inff();
                top = fmaxf(top, s[u][r]);
            }
        top = groups_max(top);
        const float m_new = fmaxf(m_run, top), m_sub = m_new == -__builtin_inff() ? 0.0f : m_new;
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_sub);
        m_run = m_new;
        float sum = 0.0f;
        bf8 ph[2], pl[2];
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const float p = __builtin_amdgcn_exp2f(s[u][r] - m_sub);
                sum += p;
                const __bf16 hi = (__bf16)p;
                ph[u >> 1][4 * (u & 1) + r] = hi, pl[u >> 1][4 * (u & 1) + r] = (__bf16)(p - (float)hi);
            }
        l_run = l_run * alpha + sum;
#pragma unroll
        for (int i = 0; i < NV; i++) o[i] *= alpha;
#pragma unroll
        for (int u = 0; u < 2; u++)
#pragma unroll
            for (int i = 0; i < NV; i++) {
                const bf4 v0 = *reinterpret_cast<const bf4*>(&vs[(16 * i + l16) * LDV + 32 * u + 4 * g]);
                const bf4 v1 = *reinterpret_cast<const bf4*>(&vs[(16 * i + l16) * LDV + 32 * u + 16 + 4 * g]);
                const bf8 v = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl[u], o[i], 0, 0, 0);
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph[u], o[i], 0, 0, 0);
            }
    }
    const float inv = 1.0f / groups_sum(l_run);
    if (jq < a.n) {
        uint16_t* out = a.out + (size_t)jq * a.ldo;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const uint32_t d = 16 * i + 4 * g;
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (d + r < a.vdim) put(out + h * a.vdim + d + r, o[i][r] * inv);
        }
        if (h + 1 == a.heads)
            for (uint32_t e = a.heads * a.vdim + g; e < a.kp; e += 4) put(out + e, 0.0f);
    }
}

bool shape_ok(const LatentShape& s) {
    return s.heads > 0 && s.dim > 0 && s.rot > 0 && s.rot % 2u == 0 && s.vdim > 0 && s.rank > 0 && s.rank_p % 32u == 0 && s.rank_p >= s.rank && s.rot_p % 32u == 0 &&
           s.rot_p >= s.rot && s.row() % 64u == 0 && s.rank_p <= 2048u;
}

template <int NS, int NV>
hipError_t run_prefill(const PrefillArgs& a, const Launch& L) {
    return launch_kernel(L, kFamOther, latent_prefill_kernel<NS, NV>, dim3(a.heads, (a.n + 63u) / 64u), dim3(256), a);
}
template <int NS>
hipError_t run_prefill_nv(const PrefillArgs& a, uint32_t dvp, const Launch& L) {
    switch (dvp) {
        case 32: return run_prefill<NS, 2>(a, L);
        case 64: return run_prefill<NS, 4>(a, L);
        case 128: return run_prefill<NS, 8>(a, L);
        default: return hipErrorInvalidValue;
    }
}

}  // namespace

hipError_t launch_latent_absorb(const LatentShape& s, const LatentWeights& w, const float* proj, uint32_t ldp, void* cache, float* qa, uint32_t n,
                                uint32_t pos0, const uint32_t* d_pos, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!shape_ok(s) || ldp < s.heads * (s.dim + s.rot) + s.rank + s.rot || (!d_pos && (uint64_t)pos0 + n > s.max_seq)) return hipErrorInvalidValue;
    const AbsorbArgs a{s, w, proj, ldp, pos0, d_pos, cache, qa};
    const dim3 grid(s.heads * ((s.rank_p + kSlab - 1u) / kSlab) + 1u, n);
    return s.f32 ? launch_kernel(L, kFamOther, latent_absorb_kernel<float>, grid, dim3(256), a)
                 : launch_kernel(L, kFamOther, latent_absorb_kernel<uint16_t>, grid, dim3(256), a);
}

hipError_t launch_latent_rope(const LatentShape& s, const LatentWeights& w, const float* proj, uint32_t ldp, void* cache, uint16_t* q, uint32_t dqp,
                              uint32_t n, uint32_t pos0, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!shape_ok(s) || s.f32 || dqp < s.dim + s.rot || ldp < s.heads * (s.dim + s.rot) + s.rank + s.rot || (uint64_t)pos0 + n > s.max_seq)
        return hipErrorInvalidValue;
    return launch_kernel(L, kFamOther, latent_rope_kernel, dim3(n), dim3(256), AbsorbArgs{s, w, proj, ldp, pos0, nullptr, cache, nullptr}, q, dqp);
}

uint32_t latent_attention_splits(const LatentShape& s, uint32_t n) {
    uint32_t splits = (s.max_seq + kChunk - 1u) / kChunk;
    if (splits > kMaxSplits) splits = kMaxSplits;
    if (n > 1) {  // many tokens fill the chip by themselves
        const uint32_t want = (1024u + n * ((s.heads + 7u) / 8u) - 1u) / (n * ((s.heads + 7u) / 8u));
        if (want < splits) splits = want;
    }
    return splits > 0 ? splits : 1u;
}

size_t latent_attention_scratch_floats(const LatentShape& s, uint32_t n) {
    return (size_t)n * s.heads * latent_attention_splits(s, n) * (s.rank_p + 4u);
}

hipError_t launch_latent_attention(const LatentShape& s, const LatentWeights& w, const float* qa, const void* cache, float* scratch, uint32_t n,
                                   uint32_t pos0, const uint32_t* d_pos, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!shape_ok(s) || (!d_pos && (uint64_t)pos0 + n > s.max_seq) || ldo < kp || kp < s.heads * s.vdim) return hipErrorInvalidValue;
    const uint32_t splits = latent_attention_splits(s, n);
    const AttendArgs a{s, qa, cache, scratch, pos0, splits, d_pos};
    auto attend = [&](auto hg, auto np) {
        constexpr int HG = decltype(hg)::value, NP = decltype(np)::value;
        const dim3 grid(splits, (s.heads + HG - 1u) / HG, n);
        const uint32_t lds = HG * s.row() * 4u, staged = lds + kChunk * s.row() * (s.f32 ? 4u : 2u);
        if constexpr (NP <= 2) {  // (longer rows do not fit)
            auto go = [&](auto kernel) {
                if (staged > 56u * 1024u) {
                    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kStageBytes);
                    if (e != hipSuccess) return e;
                }
                return launch_kernel_lds(L, kFamOther, kernel, grid, dim3(256), staged, a);
            };
            if (staged <= kStageBytes) return s.f32 ? go(latent_attend_kernel<HG, NP, true, float>) : go(latent_attend_kernel<HG, NP, true, uint16_t>);
        }
        return s.f32 ? launch_kernel_lds(L, kFamOther, latent_attend_kernel<HG, NP, false, float>, grid, dim3(256), lds, a)
                     : launch_kernel_lds(L, kFamOther, latent_attend_kernel<HG, NP, false, uint16_t>, grid, dim3(256), lds, a);
    };
    auto with_pairs = [&](auto hg) {
        if (s.rank_p <= 512u) return attend(hg, std::integral_constant<int, 1>{});
        if (s.rank_p <= 1024u) return attend(hg, std::integral_constant<int, 2>{});
        return attend(hg, std::integral_constant<int, 4>{});
    };
    // LDS holds the queries of a group of heads: eight while they leave room for a second workgroup
    hipError_t e = n == 1 && s.heads <= 16u ? with_pairs(std::integral_constant<int, 2>{})  // one token: more workgroups with less to do
                   : n > 1 && s.row() <= 1024u ? with_pairs(std::integral_constant<int, 8>{})
                                                : with_pairs(std::integral_constant<int, 4>{});
    if (e != hipSuccess) return e;
    const MergeArgs m{s, scratch, pos0, splits, d_pos, w.uv, out, ldo, kp};
    const dim3 grid(s.heads, n, n == 1 ? 4 : 1);
    return out_f32 ? launch_kernel_lds(L, kFamOther, latent_merge_kernel<float>, grid, dim3(256), s.rank_p * 4u, m)
                   : launch_kernel_lds(L, kFamOther, latent_merge_kernel<uint16_t>, grid, dim3(256), s.rank_p * 4u, m);
}

bool latent_prefill_shape(uint32_t dim, uint32_t rot, uint32_t vdim, uint32_t* dqp, uint32_t* dvp) {
    const uint32_t q = dim + rot;
    if (q > 256u || vdim > 128u) return false;
    *dqp = q <= 64u ? 64u : q <= 96u ? 96u : q <= 128u ? 128u : q <= 192u ? 192u : 256u;
    *dvp = vdim <= 32u ? 32u : vdim <= 64u ? 64u : 128u;
    return true;
}

hipError_t launch_latent_prefill(const LatentShape& s, const uint16_t* q, const uint16_t* kx, uint32_t ldk, const uint16_t* vt, uint32_t ldv, uint32_t dqp,
                                 uint32_t dvp, uint32_t n, uint32_t pos0, uint16_t* out, uint32_t ldo, uint32_t kp, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!shape_ok(s) || s.f32 || ldv % 64u || ldv < pad_to(pos0 + n, 64u) || (uint64_t)pos0 + n > s.max_seq || dvp < s.vdim || dqp < s.dim + s.rot || ldk < s.heads * dqp || ldk % 8u || ldo < kp ||
        kp < s.heads * s.vdim)
        return hipErrorInvalidValue;
    const PrefillArgs a{q, kx, vt, ldk, ldv, n, pos0, s.heads, s.vdim, s.scale * kLog2e, out, ldo, kp};
    switch (dqp) {
        case 64: return run_prefill_nv<2>(a, dvp, L);
        case 96: return run_prefill_nv<3>(a, dvp, L);
        case 128: return run_prefill_nv<4>(a, dvp, L);
        case 192: return run_prefill_nv<6>(a, dvp, L);
        case 256: return run_prefill_nv<8>(a, dvp, L);
        default: return hipErrorInvalidValue;
    }
}

}  // namespace wick_rocm
