// Grouped-query attention over a sliding window, with rotary positions on part of a head, capped scores and an output gate.
//
// The cache is a ring of positions: keys row by row, values in tiles of 64 positions with the positions side by side, so that a weighted sum
// reads them in vectors along the positions and a tile is an operand of the matrix cores as it lies in memory.
//   a few queries  (decode steps, short portions, the f32 model) split over the window, all arithmetic f32.  A step turns its query and
//                  its key inside the launch, appends key and value itself and uses them from the projection, whoever stored them;
//   many queries   64 queries x 64 positions at a time on the matrix cores, tiles that no query of the workgroup sees are skipped.
// Softmax is streamed in f32.
#include "window_attend.h"

namespace wick_rocm {

namespace {

struct StoreArgs {
    WindowShape s;
    WindowProj w;
    void *kc, *vc;
    uint32_t n, pos0;
};

// Workgroup: eight neighbouring positions (a vector of the value tiles) of one key / value head.
template <typename CT>
__global__ __launch_bounds__(256) void window_store_kernel(StoreArgs a) {
    const WindowShape& s = a.s;
    const uint32_t g = blockIdx.y, p0 = (a.pos0 / 8u + blockIdx.x) * 8u, end = a.pos0 + a.n;
    const uint32_t slot0 = p0 % s.slots;  // (slots is a multiple of 64: the eight do not wrap)
    CT *kc = static_cast<CT*>(a.kc), *vc = static_cast<CT*>(a.vc);
    const uint32_t pairs = s.dqp / 2u;
    for (uint32_t i = threadIdx.x; i < 8u * pairs; i += 256) {
        const uint32_t j = i / pairs, e = 2u * (i % pairs), p = p0 + j;
        if (p < a.pos0 || p >= end) continue;
        const float2 v = rotated_pair(a.w.p + (size_t)(p - a.pos0) * a.w.ldp + a.w.k_at + g * s.dqp, e, a.w.rope, s.rot, p);
        CT* o = kc + ((size_t)(slot0 + j) * s.kv_heads + g) * s.dqp + e;
        put(o, v.x), put(o + 1, v.y);
    }
    const bool whole = p0 >= a.pos0 && p0 + 8u <= end;
    for (uint32_t d = threadIdx.x; d < s.dvp; d += 256) {
        CT* o = vc + (((size_t)(slot0 / kTile) * s.kv_heads + g) * s.dvp + d) * kTile + slot0 % kTile;
        float v[8];
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) {
            const uint32_t p = p0 + j;
            v[j] = p >= a.pos0 && p < end ? a.w.p[(size_t)(p - a.pos0) * a.w.ldp + a.w.v_at + g * s.dvp + d] : 0.0f;
        }
        if (whole && sizeof(CT) == 2) {
            bf8 b;
#pragma unroll
            for (int j = 0; j < 8; j++) b[j] = (__bf16)v[j];
            *reinterpret_cast<bf8*>(o) = b;
        } else {
#pragma unroll
            for (uint32_t j = 0; j < 8; j++)
                if (p0 + j >= a.pos0 && p0 + j < end) put(o + j, v[j]);
        }
    }
}

template <int HG, int NP, typename CT>
__global__ __launch_bounds__(256) void window_attend_kernel(AttendArgs a) {
    extern __shared__ __align__(16) float qs[];
    window_attend_block<HG, NP, CT>(a, blockIdx.x, blockIdx.y, blockIdx.z, qs);
}

// Workgroup (head, token): the partials of the splits, then the gate.
__global__ __launch_bounds__(256) void window_merge_kernel(WindowMerge a, void* out, uint32_t ldo, uint32_t kp, bool out_f32) {
    __shared__ float wts[kMaxSplits];
    const WindowShape& s = a.s;
    const uint32_t h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, stride = s.dvp + 4u;
    auto store = [&](uint32_t e, float v) {
        if (out_f32) static_cast<float*>(out)[(size_t)t * ldo + e] = v;
        else put(static_cast<uint16_t*>(out) + (size_t)t * ldo + e, v);
    };
    const float* parts = a.part + ((size_t)t * s.heads + h) * a.splits * stride;
    // what the first pass needs is requested before the totals are known (behind the last active partial lies something older)
    const uint32_t d0 = tid < s.vdim ? tid : 0u;
    float pre[8];
#pragma unroll
    for (uint32_t i = 0; i < 8; i++) pre[i] = parts[(size_t)(i < a.splits ? i : 0u) * stride + 4 + d0];
    const float gate0 = a.w.p[(size_t)t * a.w.ldp + a.w.g_at + h * s.dvp + d0];
    const float m_raw = parts[(size_t)(tid < a.splits ? tid : 0u) * stride], l_raw = parts[(size_t)(tid < a.splits ? tid : 0u) * stride + 1];
    const uint32_t pos = (a.d_pos ? *a.d_pos : a.pos0) + t;
    if (pos >= s.max_seq) return;
    uint32_t tile0, active = s.window_tiles(pos, tile0);
    active = active < a.splits ? active : a.splits;
    if (tid < 64) {
        const bool on = tid < active;
        const float m_i = on ? m_raw : -__builtin_inff(), m = wave_max_f32(m_i), w = on ? expf(m_i - m) : 0.0f;
        wts[tid] = w / wave_sum_f32(on ? l_raw * w : 0.0f);
    }
    __syncthreads();
    for (uint32_t d = tid; d < s.vdim; d += 256) {
        float v = 0.0f;
#pragma unroll
        for (uint32_t i = 0; i < 8; i++)
            if (i < active) v += (d == tid ? pre[i] : parts[(size_t)i * stride + 4 + d]) * wts[i];
        for (uint32_t i = 8; i < active; i++) v += parts[(size_t)i * stride + 4 + d] * wts[i];
        const float gate = d == tid ? gate0 : a.w.p[(size_t)t * a.w.ldp + a.w.g_at + h * s.dvp + d];
        store( h * s.vdim + d, v * sigmoidf(gate));
    }
    if (h + 1 == s.heads)
        for (uint32_t e = s.heads * s.vdim + tid; e < kp; e += 256) store( e, 0.0f);
}

// ---- many queries --------------------------------------------------------------------------------------------------------------
struct PrefillArgs {
    WindowShape s;
    WindowProj w;
    const uint16_t *kc, *vc;
    uint32_t n, pos0;
    float scale, cap, cap_inv;  // in units of log 2: a score is scaled, then, with a cap, cap * tanh of half of score * cap_inv
    uint16_t* out;
    uint32_t ldo, kp;
};

// Workgroup: one head, 64 queries, 16 per wave; 64 positions at a time through LDS, the next tile's loads in flight meanwhile.
//   scores transposed: S^T[key][query], A = K, B = Q^T (the turned query as two bfloat16 terms): lane l holds keys 4 (l / 16) + r of
//   query l % 16; values transposed: O^T[d][query] += V^T[d][key] P[key][query]: the weights go from one product into the next in the
//   registers they are in -- slot j of lane group g stands for key 4 g + j of a 16-key sub-tile (j < 4) or of the next one (j >= 4) in
//   both operands.  The weights enter as two bfloat16 terms, so they keep 16 bits.
// BOUNDED: the cap itself serves as the maximum of every row's scores.
template <int NS, int NV, bool BOUNDED>
__global__ __launch_bounds__(256) void window_prefill_kernel(PrefillArgs a) {
    constexpr uint32_t DQ = 32 * NS, DV = 16 * NV, LDK = DQ + 8, LDV = 72;
    __shared__ __align__(16) uint16_t ks[64 * LDK], vs[DV * LDV];
    const WindowShape& s = a.s;
    const uint32_t h = blockIdx.x, kvh = h / (s.heads / s.kv_heads), qblocks = (a.n + 63u) / 64u, j0 = (qblocks - 1u - blockIdx.y) * 64u;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4, ring = s.slots / kTile;
    const uint32_t jq = j0 + 16u * wave + l16, jl = jq < a.n ? jq : a.n - 1u, pq = a.pos0 + jl, lo_key = s.first_seen(pq);
    const uint32_t wg_last = a.pos0 + (j0 + 63u < a.n ? j0 + 63u : a.n - 1u), tile0 = s.first_seen(a.pos0 + j0) / kTile;
    const uint32_t wave_first = a.pos0 + j0 + 16u * wave, wave_last = wave_first + 15u < wg_last ? wave_first + 15u : wg_last;
    const uint32_t wave_lo = s.first_seen(wave_first), wave_lo_last = s.first_seen(wave_last);
    const bool active = j0 + 16u * wave < a.n;
    constexpr int KP = 64 * (DQ / 8) / 256, VP = DV * 8 / 256;
    u4 kr[KP], vr[VP];
    auto fetch = [&](uint32_t tile) {
        const uint32_t slot = tile % ring;
#pragma unroll
        for (int i = 0; i < KP; i++) {
            const uint32_t c = tid + 256u * i, r = c / (DQ / 8), ch = c % (DQ / 8);
            kr[i] = *reinterpret_cast<const u4*>(a.kc + ((size_t)(slot * kTile + r) * s.kv_heads + kvh) * DQ + 8u * ch);
        }
        const uint16_t* v = a.vc + ((size_t)slot * s.kv_heads + kvh) * DV * kTile;
#pragma unroll
        for (int i = 0; i < VP; i++) vr[i] = *reinterpret_cast<const u4*>(v + 8u * (tid + 256u * i));
    };
    fetch(tile0);
    bf8 qh[NS], ql[NS];
    {
        const float* q = a.w.p + (size_t)jl * a.w.ldp + a.w.q_at + h * DQ;
#pragma unroll
        for (int i = 0; i < NS; i++)
#pragma unroll
            for (int k = 0; k < 4; k++) {
                const float2 v = rotated_pair(q, 32u * i + 8u * g + 2u * k, a.w.rope, s.rot, pq);
                qh[i][2 * k] = (__bf16)v.x, qh[i][2 * k + 1] = (__bf16)v.y;
                ql[i][2 * k] = (__bf16)(v.x - (float)qh[i][2 * k]), ql[i][2 * k + 1] = (__bf16)(v.y - (float)qh[i][2 * k + 1]);
            }
    }
    v4f o[NV];
#pragma unroll
    for (int i = 0; i < NV; i++) o[i] = v4f{0.f, 0.f, 0.f, 0.f};
    float m_run = -__builtin_inff(), l_run = 0.0f;
    for (uint32_t tile = tile0; tile * kTile <= wg_last; tile++) {
        const uint32_t t0 = tile * kTile;
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
        if (t0 + kTile <= wg_last) fetch(tile + 1u);
        if (!active || t0 > wave_last || t0 + kTile <= wave_lo) continue;
        v4f sc[4];
#pragma unroll
        for (int u = 0; u < 4; u++) sc[u] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NS; i++) {
            bf8 k[4];
#pragma unroll
            for (int u = 0; u < 4; u++) k[u] = *reinterpret_cast<const bf8*>(&ks[(16 * u + l16) * LDK + 32 * i + 8 * g]);
#pragma unroll
            for (int u = 0; u < 4; u++) sc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[u], ql[i], sc[u], 0, 0, 0);
#pragma unroll
            for (int u = 0; u < 4; u++) sc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[u], qh[i], sc[u], 0, 0, 0);
        }
        const bool masked = t0 + 63u > wave_first || t0 < wave_lo_last;
        auto out_of_sight = [&](int u, int r) {
            const uint32_t p = t0 + 16u * u + 4u * g + r;
            return masked && (p > pq || p < lo_key);
        };
        float m_sub = 0.0f;
        if constexpr (BOUNDED) {  // cap tanh(x) - cap = -2 cap / (1 + exp(2 x))
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const float v = -2.0f * a.cap * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(sc[u][r] * a.cap_inv));
                    sc[u][r] = out_of_sight(u, r) ? -__builtin_inff() : v;
                }
        } else {
            float top = -__builtin_inff();
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    float v = sc[u][r] * a.scale;
                    if (a.cap > 0.0f) v = fmaf(-2.0f * a.cap, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(sc[u][r] * a.cap_inv)), a.cap);
                    if (out_of_sight(u, r)) v = -__builtin_inff();
                    sc[u][r] = v;
                    top = fmaxf(top, v);
                }
            top = groups_max(top);
            const float m_new = fmaxf(m_run, top);
            m_sub = m_new == -__builtin_inff() ? 0.0f : m_new;
            const float alpha = __builtin_amdgcn_exp2f(m_run - m_sub);
            m_run = m_new, l_run *= alpha;
#pragma unroll
            for (int i = 0; i < NV; i++) o[i] *= alpha;
        }
        bf8 ph[2], pl[2];
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const float p = __builtin_amdgcn_exp2f(sc[u][r] - m_sub);
                l_run += p;
                const __bf16 hi = (__bf16)p;
                ph[u >> 1][4 * (u & 1) + r] = hi, pl[u >> 1][4 * (u & 1) + r] = (__bf16)(p - (float)hi);
            }
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
        uint16_t* out = a.out + (size_t)jq * a.ldo + h * s.vdim;
        const float* gate = a.w.p + (size_t)jq * a.w.ldp + a.w.g_at + h * DV;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const uint32_t d = 16 * i + 4 * g;
            const v4f z = *reinterpret_cast<const v4f*>(gate + d);
            v4f y;
#pragma unroll
            for (int r = 0; r < 4; r++) y[r] = o[i][r] * inv * sigmoid_hw(z[r]);
            if (s.vdim % 4u == 0) {
                const bf4 b = {(__bf16)y[0], (__bf16)y[1], (__bf16)y[2], (__bf16)y[3]};
                if (d < s.vdim) *reinterpret_cast<bf4*>(out + d) = b;
            } else {
#pragma unroll
                for (int r = 0; r < 4; r++)
                    if (d + r < s.vdim) put(out + d + r, y[r]);
            }
        }
        if (h + 1 == s.heads)
            for (uint32_t e = s.heads * s.vdim + g; e < a.kp; e += 4) a.out[(size_t)jq * a.ldo + e] = 0;
    }
}

}  // namespace

uint32_t window_slots(uint32_t window, uint32_t portion, uint32_t max_seq) {
    const uint64_t all = pad_to(max_seq, kTile), need = window ? pad_to(window - 1u + portion, kTile) : all;
    return (uint32_t)(need < all ? need : all);
}

bool window_prefill_shape(uint32_t dim, uint32_t vdim) { return dim <= 256u && vdim <= 256u; }

void window_pads(uint32_t dim, uint32_t vdim, uint32_t* dqp, uint32_t* dvp) {
    auto pad = [](uint32_t d) { return d <= 64u ? 64u : d <= 96u ? 96u : d <= 128u ? 128u : d <= 256u ? 256u : pad_to(d, 32u); };
    *dqp = pad(dim), *dvp = pad(vdim);
}

size_t window_attention_scratch_floats(const WindowShape& s, uint32_t n) { return (size_t)n * s.heads * attend_splits(s, n) * (s.dvp + 4u); }

hipError_t launch_window_store(const WindowShape& s, const WindowProj& w, void* kc, void* vc, uint32_t n, uint32_t pos0, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!window_shape_ok(s, w, n, pos0, true)) return hipErrorInvalidValue;
    const dim3 grid((pos0 + n + 7u) / 8u - pos0 / 8u, s.kv_heads);
    const StoreArgs a{s, w, kc, vc, n, pos0};
    return s.f32 ? launch_kernel(L, kFamOther, window_store_kernel<float>, grid, dim3(256), a)
                 : launch_kernel(L, kFamOther, window_store_kernel<uint16_t>, grid, dim3(256), a);
}

hipError_t launch_window_attention(const WindowShape& s, const WindowProj& w, void* kc, void* vc, float* scratch, uint32_t n, uint32_t pos0,
                                   const uint32_t* d_pos, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L) {
    if (n == 0) return hipSuccess;
    AttendPlan p;
    if (!plan_attend(s, w, kc, vc, scratch, n, pos0, d_pos, out, ldo, kp, out_f32, p)) return hipErrorInvalidValue;
    const dim3 grid(p.a.splits, p.blocks_y, n);
    const hipError_t e = attend_sizes(s, n, [&](auto hg, auto np) {
        constexpr int HG = decltype(hg)::value, NP = decltype(np)::value;
        return s.f32 ? launch_kernel_lds(L, kFamOther, window_attend_kernel<HG, NP, float>, grid, dim3(256), p.lds, p.a)
                     : launch_kernel_lds(L, kFamOther, window_attend_kernel<HG, NP, uint16_t>, grid, dim3(256), p.lds, p.a);
    });
    if (e != hipSuccess || p.a.splits == 1u) return e;
    return launch_window_merge(p.merge(), n, out, ldo, kp, out_f32, L);
}

hipError_t launch_window_merge(const WindowMerge& m, uint32_t n, void* out, uint32_t ldo, uint32_t kp, bool out_f32, const Launch& L) {
    if (!m.part || m.splits == 0 || m.splits > kMaxSplits || ldo < kp || kp < m.s.heads * m.s.vdim) return hipErrorInvalidValue;
    return launch_kernel(L, kFamOther, window_merge_kernel, dim3(m.s.heads, n), dim3(256), m, out, ldo, kp, out_f32);
}

bool window_merge_foldable(const WindowMerge& m) { return m.d_pos && m.splits > 1u && m.splits <= 32u && m.s.vdim % 4u == 0; }

hipError_t launch_window_prefill(const WindowShape& s, const WindowProj& w, const void* kc, const void* vc, uint32_t n, uint32_t pos0, uint16_t* out,
                                 uint32_t ldo, uint32_t kp, const Launch& L) {
    if (n == 0) return hipSuccess;
    if (!window_shape_ok(s, w, n, pos0, true) || s.f32 || ldo < kp || kp < s.heads * s.vdim || ldo % 4u) return hipErrorInvalidValue;
    PrefillArgs a{s, w, static_cast<const uint16_t*>(kc), static_cast<const uint16_t*>(vc), n, pos0, s.scale * kLog2e, 0.0f, 0.0f, out, ldo, kp};
    if (s.softcap > 0.0f) a.cap = s.softcap * kLog2e, a.cap_inv = 2.0f * kLog2e * s.scale / s.softcap;  // tanh(x) = 1 - 2 / (1 + exp(2 x))
    const bool bounded = s.softcap > 0.0f && a.cap <= 48.0f;  // weights from exp2(-2 cap) on: far from the end of the f32 range
    const dim3 grid(s.heads, (n + 63u) / 64u);
    auto go = [&](auto ns) {
        constexpr int NS = decltype(ns)::value;
        auto run = [&](auto nv) {
            constexpr int NV = decltype(nv)::value;
            return bounded ? launch_kernel(L, kFamOther, window_prefill_kernel<NS, NV, true>, grid, dim3(256), a)
                           : launch_kernel(L, kFamOther, window_prefill_kernel<NS, NV, false>, grid, dim3(256), a);
        };
        switch (s.dvp) {
            case 64: return run(std::integral_constant<int, 4>{});
            case 96: return run(std::integral_constant<int, 6>{});
            case 128: return run(std::integral_constant<int, 8>{});
            case 256: return run(std::integral_constant<int, 16>{});
            default: return hipErrorInvalidValue;
        }
    };
    switch (s.dqp) {
        case 64: return go(std::integral_constant<int, 2>{});
        case 96: return go(std::integral_constant<int, 3>{});
        case 128: return go(std::integral_constant<int, 4>{});
        case 256: return go(std::integral_constant<int, 8>{});
        default: return hipErrorInvalidValue;
    }
}

}  // namespace wick_rocm
