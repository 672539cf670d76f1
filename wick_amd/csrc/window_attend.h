// Device code of windowed attention for a few queries, shared by the launches it appears in.  Not installed.
#pragma once

#include <type_traits>

#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));
typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
typedef uint32_t u4 __attribute__((ext_vector_type(4)));

constexpr uint32_t kTile = kWindowTile;
constexpr uint32_t kMaxSplits = 64;  // workgroups along the window
constexpr uint32_t kSlab = 256;      // value coordinates of a workgroup
constexpr float kLog2e = 1.44269504088896340736f;

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(uint16_t* p, float v) { *p = __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ float as_cached(float v, const float*) { return v; }
__device__ __forceinline__ float as_cached(float v, const uint16_t*) { return (float)(__bf16)v; }
__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }

__device__ __forceinline__ void widen8(u4 w, float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 4; i++) v[2 * i] = __uint_as_float(w[i] << 16), v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
}
__device__ __forceinline__ void load8(const uint16_t* p, float (&v)[8]) { widen8(*reinterpret_cast<const u4*>(p), v); }
__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
    const v4f a = *reinterpret_cast<const v4f*>(p), b = *reinterpret_cast<const v4f*>(p + 4);
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = a[i], v[4 + i] = b[i];
}

// Coordinates e, e + 1 (e even) of a head at `pos`, turned when they are a pair that turns.
__device__ __forceinline__ float2 rotated_pair(const float* head, uint32_t e, const float* rope, uint32_t rot, uint32_t pos) {
    const float2 v = *reinterpret_cast<const float2*>(head + e);
    if (e >= rot) return v;
    const float2 cs = *reinterpret_cast<const float2*>(rope + (size_t)pos * rot + e);
    return float2{v.x * cs.x - v.y * cs.y, v.y * cs.x + v.x * cs.y};
}

// ---- a few queries ------------------------------------------------------------------------------------------------------------
struct AttendArgs {
    WindowShape s;
    WindowProj w;
    void *kc, *vc;
    float* part;          // WindowMerge
    uint32_t pos0, splits, hgroups;
    const uint32_t* d_pos;   // non-null: a step
    void* out;               // splits == 1: the result itself
    uint32_t ldo, kp;
    bool out_f32;
};

__device__ __forceinline__ void put_out(const AttendArgs& a, uint32_t t, uint32_t e, float v) {
    if (a.out_f32) static_cast<float*>(a.out)[(size_t)t * a.ldo + e] = v;
    else put(static_cast<uint16_t*>(a.out) + (size_t)t * a.ldo + e, v);
}

// One workgroup of 256 threads: (split, key / value head x group of HG query heads x slab of value coordinates, token).  qs: LDS,
// [HG][dqp] | the step's key [dqp].  Scores: four lanes a key; values: eight
// lanes a coordinate, eight positions each.
template <int HG, int NP, typename CT>
__device__ __forceinline__ void window_attend_block(const AttendArgs& a, uint32_t split, uint32_t which, uint32_t t, float* qs) {
    __shared__ __align__(16) float sc[HG][kTile];
    __shared__ float corr[HG];
    const WindowShape& s = a.s;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t slabs = (s.dvp + kSlab - 1u) / kSlab, slab = which % slabs, hgroup = which / slabs % a.hgroups, g = which / (slabs * a.hgroups);
    const uint32_t ratio = s.heads / s.kv_heads, h0 = g * ratio + hgroup * HG, nh = ratio - hgroup * HG < (uint32_t)HG ? ratio - hgroup * HG : (uint32_t)HG;
    const bool step = a.d_pos != nullptr;
    const uint32_t pos = (step ? *a.d_pos : a.pos0) + t;
    if (pos >= s.max_seq) return;  // the host checks by-value positions; a device-side one past the cache is dropped
    const float* proj = a.w.p + (size_t)t * a.w.ldp;
    uint32_t tile0;
    const uint32_t tiles = s.window_tiles(pos, tile0), first = s.first_seen(pos), ring = s.slots / kTile;
    if (split >= tiles) return;  // the merge derives the number of partials from pos as well
    CT *kc = static_cast<CT*>(a.kc), *vc = static_cast<CT*>(a.vc);
    const uint32_t key = tid >> 2, l4 = tid & 3u, l8 = tid & 7u, row = tid >> 3;

    // the first tile's keys and values are requested before the queries
    constexpr int KA = sizeof(CT) == 2 ? 4 : 1;  // pieces of a key in flight per lane
    u4 ka[KA], va[NP];
    auto key_row = [&](uint32_t tile) { return kc + ((size_t)((tile % ring) * kTile + key) * s.kv_heads + g) * s.dqp; };
    auto value_row = [&](uint32_t tile, uint32_t d) { return vc + (((size_t)(tile % ring) * s.kv_heads + g) * s.dvp + d) * kTile + 8u * l8; };
    auto request = [&](uint32_t tile) {
        if constexpr (sizeof(CT) == 2) {
            const CT* kr = key_row(tile);
#pragma unroll
            for (int i = 0; i < KA; i++) ka[i] = *reinterpret_cast<const u4*>(kr + (8u * l4 + 32u * i < s.dqp ? 8u * l4 + 32u * i : 0u));
#pragma unroll
            for (int i = 0; i < NP; i++) {
                const uint32_t d = slab * kSlab + row + 32u * i;
                va[i] = *reinterpret_cast<const u4*>(value_row(tile, d < s.dvp ? d : 0u));
            }
        }
    };
    request(tile0 + split);

    const uint32_t last_tile = pos / kTile;
    const bool has_new = step && (last_tile - tile0) % a.splits == split;  // this workgroup meets the step's own position
    float* knew = qs + HG * s.dqp;
    for (uint32_t i = tid; i < (HG + 1u) * (s.dqp / 2u); i += 256) {
        const uint32_t h = i / (s.dqp / 2u), e = 2u * (i % (s.dqp / 2u));
        float2 v = {0.0f, 0.0f};
        if (h == (uint32_t)HG) {
            if (!has_new) continue;
            v = rotated_pair(proj + a.w.k_at + g * s.dqp, e, a.w.rope, s.rot, pos);
            v.x = as_cached(v.x, kc), v.y = as_cached(v.y, kc);
            if (hgroup == 0 && slab == 0) {
                CT* o = kc + ((size_t)(pos % s.slots) * s.kv_heads + g) * s.dqp + e;
                put(o, v.x), put(o + 1, v.y);
            }
        } else if (h < nh) {
            v = rotated_pair(proj + a.w.q_at + (h0 + h) * s.dqp, e, a.w.rope, s.rot, pos);
        }
        qs[h * s.dqp + e] = v.x, qs[h * s.dqp + e + 1] = v.y;
    }
    __syncthreads();

    float acc[NP][HG], m_run = -__builtin_inff(), l_run = 0.0f;
#pragma unroll
    for (int i = 0; i < NP; i++)
#pragma unroll
        for (int h = 0; h < HG; h++) acc[i][h] = 0.0f;

    for (uint32_t c = split; c < tiles; c += a.splits) {
        const uint32_t tile = tile0 + c, p = tile * kTile + key;
        const bool is_new = step && p == pos, seen = p >= first && p <= pos;
        if (c != split) request(tile);
        float dot[HG];
#pragma unroll
        for (int h = 0; h < HG; h++) dot[h] = 0.0f;
        const CT* kr = key_row(tile);
        auto piece = [&](uint32_t at, float (&kv)[8]) {
            if (is_new) load8(knew + at, kv);
#pragma unroll
            for (int h = 0; h < HG; h++) {
                const v4f q0 = *reinterpret_cast<const v4f*>(qs + h * s.dqp + at), q1 = *reinterpret_cast<const v4f*>(qs + h * s.dqp + at + 4);
#pragma unroll
                for (int i = 0; i < 4; i++) dot[h] = fmaf(q0[i], kv[i], fmaf(q1[i], kv[4 + i], dot[h]));
            }
        };
        uint32_t at = 8u * l4;
        if constexpr (sizeof(CT) == 2) {
#pragma unroll
            for (int i = 0; i < KA; i++, at += 32u)
                if (at < s.dqp) {
                    float kv[8];
                    widen8(ka[i], kv);
                    piece(at, kv);
                }
        }
        for (; at < s.dqp; at += 32u) {
            float kv[8];
            load8(kr + at, kv);
            piece(at, kv);
        }
#pragma unroll
        for (int h = 0; h < HG; h++) {
            float d = group_sum<4>(dot[h]) * s.scale;
            if (s.softcap > 0.0f) d = s.softcap * tanhf(d / s.softcap);
            if (l4 == 0) sc[h][key] = seen ? d : -__builtin_inff();
        }
        __syncthreads();
        if (wave < (uint32_t)HG) {  // one wave a head; a tile of the window has at least one position that is seen: finite
            const float v = sc[wave][lane], m_new = fmaxf(m_run, wave_max_f32(v));
            const float e = expf(v - m_new), f = expf(m_run - m_new);
            sc[wave][lane] = e;
            l_run = l_run * f + wave_sum_f32(e);
            m_run = m_new;
            if (lane == 0) corr[wave] = f;
        }
        __syncthreads();
        const bool meets = step && pos / 8u == (tile * kTile) / 8u + l8;  // this lane's eight positions contain the step's own
#pragma unroll
        for (int i = 0; i < NP; i++) {
            const uint32_t d = slab * kSlab + row + 32u * i;
            if (d < s.dvp) {
                float v[8];
                if constexpr (sizeof(CT) == 2) widen8(va[i], v);
                else load8(value_row(tile, d), v);
                if (meets) {
                    const float mine = as_cached(proj[a.w.v_at + g * s.dvp + d], vc);
#pragma unroll
                    for (int j = 0; j < 8; j++)
                        if ((uint32_t)j == (pos & 7u)) v[j] = mine;
                    if (hgroup == 0) put(value_row(tile, d) + (pos & 7u), mine);
                }
#pragma unroll
                for (int h = 0; h < HG; h++) {
                    const v4f w0 = *reinterpret_cast<const v4f*>(&sc[h][8u * l8]), w1 = *reinterpret_cast<const v4f*>(&sc[h][8u * l8 + 4]);
                    float o = acc[i][h] * corr[h];
#pragma unroll
                    for (int j = 0; j < 4; j++) o = fmaf(w0[j], v[j], fmaf(w1[j], v[4 + j], o));
                    acc[i][h] = o;
                }
            }
        }
        __syncthreads();  // sc and corr are rewritten by the next tile
    }
    if (a.splits == 1u) {
        if (wave < (uint32_t)HG && lane == 0) corr[wave] = 1.0f / l_run;
        __syncthreads();
    }
    auto part_of = [&](uint32_t h) { return a.part + (((size_t)t * s.heads + h0 + h) * a.splits + split) * (s.dvp + 4u); };
    if (a.splits > 1u && slab == 0 && wave < nh && lane == 0) part_of(wave)[0] = m_run, part_of(wave)[1] = l_run;
#pragma unroll
    for (int i = 0; i < NP; i++)
#pragma unroll
        for (int h = 0; h < HG; h++) {
            const float o = group_sum<8>(acc[i][h]);
            const uint32_t d = slab * kSlab + row + 32u * i;
            if (l8 != 0 || h >= (int)nh || d >= s.vdim) continue;
            if (a.splits > 1u) part_of(h)[4 + d] = o;
            else put_out(a, t, (h0 + h) * s.vdim + d, o * corr[h] * sigmoidf(proj[a.w.g_at + (h0 + h) * s.dvp + d]));
        }
    if (a.splits == 1u && h0 + nh == s.heads && slab == 0)
        for (uint32_t e = s.heads * s.vdim + tid; e < a.kp; e += 256) put_out(a, t, e, 0.0f);
}

inline uint32_t attend_head_group(const WindowShape& s, uint32_t n) {
    const uint32_t ratio = s.heads / s.kv_heads;
    return ratio == 1u ? 1u : ratio == 2u || n == 1u ? 2u : 4u;
}

inline uint32_t attend_splits(const WindowShape& s, uint32_t n) {
    const uint32_t reach = s.window && s.window < s.max_seq ? s.window + kTile - 1u : s.max_seq;
    uint32_t splits = (reach + kTile - 1u) / kTile;
    if (splits > kMaxSplits) splits = kMaxSplits;
    if (n > 1) {  // many tokens fill the chip by themselves
        const uint32_t each = n * s.kv_heads * ((s.heads / s.kv_heads + 3u) / 4u), want = (1024u + each - 1u) / each;
        if (want < splits) splits = want;
    }
    return splits > 0 ? splits : 1u;
}

inline bool window_shape_ok(const WindowShape& s, const WindowProj& w, uint32_t n, uint32_t pos0, bool by_value) {
    const uint32_t reach = s.window ? s.window - 1u : s.max_seq;
    return s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && s.dqp >= s.dim && s.dvp >= s.vdim && s.dqp % 32u == 0 &&
           s.dvp % 32u == 0 && s.rot % 2u == 0 && s.rot <= s.dim && s.slots % kTile == 0 && (s.slots >= s.max_seq || (s.window && s.slots >= reach + n)) &&
           (w.ldp | w.q_at | w.k_at | w.v_at | w.g_at) % 4u == 0 && w.p && (!by_value || (uint64_t)pos0 + n <= s.max_seq);
}

// The launch's arguments, grid (splits, .y) and LDS; false: shapes that do not fit.
struct AttendPlan {
    AttendArgs a;
    uint32_t blocks_y, lds;
    WindowMerge merge() const { return WindowMerge{a.s, a.w, a.part, a.pos0, a.splits, a.d_pos}; }
};
inline bool plan_attend(const WindowShape& s, const WindowProj& w, void* kc, void* vc, float* scratch, uint32_t n, uint32_t pos0, const uint32_t* d_pos, void* out,
                        uint32_t ldo, uint32_t kp, bool out_f32, AttendPlan& o) {
    if (!window_shape_ok(s, w, n, pos0, !d_pos) || (d_pos && n != 1) || ldo < kp || kp < s.heads * s.vdim) return false;
    const uint32_t hg = attend_head_group(s, n), ratio = s.heads / s.kv_heads, slabs = (s.dvp + kSlab - 1u) / kSlab;
    o.a = AttendArgs{s, w, kc, vc, scratch, pos0, attend_splits(s, n), (ratio + hg - 1u) / hg, d_pos, out, ldo, kp, out_f32};
    o.blocks_y = s.kv_heads * o.a.hgroups * slabs, o.lds = (hg + 1u) * s.dqp * 4u;
    return o.lds <= 56u * 1024u;
}
// go(HG, NP) with the compile-time sizes of a launch.
template <typename Go>
hipError_t attend_sizes(const WindowShape& s, uint32_t n, Go&& go) {
    auto with_values = [&](auto hg) {
        if (s.dvp <= 64u) return go(hg, std::integral_constant<int, 2>{});
        if (s.dvp <= 128u) return go(hg, std::integral_constant<int, 4>{});
        return go(hg, std::integral_constant<int, 8>{});
    };
    switch (attend_head_group(s, n)) {
        case 1: return with_values(std::integral_constant<int, 1>{});
        case 2: return with_values(std::integral_constant<int, 2>{});
        default: return with_values(std::integral_constant<int, 4>{});
    }
}

}  // namespace

}  // namespace wick_rocm
