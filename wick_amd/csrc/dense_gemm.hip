// Matrix products of a prompt for bfloat16 weights: out[t][f] = sum_k W[f][k] x[t][k] for n token rows, with what follows the product
// (bias, activation, gate, the coefficients of a recurrence) in the epilogue.
//
// Two bodies share the epilogues, because the 16 x 16 result of v_mfma_f32_16x16x32_bf16 and of v_mfma_f32_16x16x4_f32 sits in the
// same registers (lane l: column l % 16, rows 4 (l / 16) + r):
//   gemm_bf16_kernel  activations in bfloat16; WM x WN waves of (16 MT) x (16 NT) outputs, K in steps of 64 through two LDS buffers
//                     (the global loads of the next PD steps are in flight during the products of this one: a tile of a small
//                     product is alone on its CU, and a step's products are much shorter than a trip to memory; the tiles of a large one
//                     are shared by sixteen waves, which hide the trips themselves and read every operand half as often); the 16-byte
//                     chunks of an LDS row are permuted by row % 8, so that the 16 rows a fragment read touches spread over the banks;
//   gemm_f32_kernel   activations in f32, weights widened exactly: every product and sum in f32.
// Weights are the M side, so a lane ends with four consecutive features of one token: one vector store.  With TRANS the sides are
// swapped and a lane holds four consecutive tokens of one feature (a transposed result).
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));
typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
typedef uint32_t u4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float bf16_to_f32(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }

__device__ __forceinline__ void store4(float* p, v4f v) { *reinterpret_cast<v4f*>(p) = v; }
__device__ __forceinline__ void store4(uint16_t* p, v4f v) {
    bf4 b;
#pragma unroll
    for (int i = 0; i < 4; i++) b[i] = (__bf16)v[i];
    *reinterpret_cast<bf4*>(p) = b;
}

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float siluf(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float gelu_tanhf(float z) {
    // 0.5 (1 + tanh(s)) = 1 / (1 + exp(-2 s))
    const float s = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * s));
}

// ---- epilogues: (z, first feature, token row of the output, sums[, sums of the second weight]) --------------------------
struct EpiStore {
    static constexpr bool kPaired = false, kTrans = false;
    float* out;
    uint32_t ldo;
    const float* add;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f) const {
        if (add) a += *reinterpret_cast<const v4f*>(add + f);
        store4(out + (size_t)t * ldo + f, a);
    }
};
struct EpiGeluSplit {
    static constexpr bool kPaired = false, kTrans = false;
    float* out;
    uint32_t ldo;
    const float* bias;
    uint32_t split;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f) const {
        a += *reinterpret_cast<const v4f*>(bias + f);
        if (f < split) {
#pragma unroll
            for (int i = 0; i < 4; i++) a[i] = gelu_tanhf(a[i]);
        }
        store4(out + (size_t)t * ldo + f, a);
    }
};
template <typename AT>
struct EpiRelu2 {
    static constexpr bool kPaired = false, kTrans = false;
    AT* out;
    uint32_t ldo;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f) const {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float r = fmaxf(a[i], 0.0f);
            a[i] = r * r;
        }
        store4(out + (size_t)t * ldo + f, a);
    }
};
template <typename AT>
struct EpiSilu {
    static constexpr bool kPaired = true, kTrans = false;
    AT* out;
    uint32_t ldo;
    const float* row_scale;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f g, v4f u) const {
        const float s = row_scale ? row_scale[t] : 1.0f;
#pragma unroll
        for (int i = 0; i < 4; i++) g[i] = siluf(g[i]) * u[i] * s;
        store4(out + (size_t)t * ldo + f, g);
    }
};
// Rows below `split` as they are, the pairs behind them through gelu(gate) * up.
template <typename AT>
struct EpiProject {
    static constexpr bool kPaired = true, kTrans = false;
    float* out;
    uint32_t ldo, split;
    AT* act;
    uint32_t lda;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f b) const {
        const uint32_t row = 2u * (f & ~15u) + (f & 15u);  // of the first of the two
        if (row < split) {
            float* o = out + (size_t)t * ldo + row;
            store4(o, a), store4(o + 16, b);
            return;
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            if constexpr (sizeof(AT) == 2) a[i] = a[i] * sigmoid_hw(1.59576912160573071176f * (a[i] + 0.044715f * a[i] * a[i] * a[i])) * b[i];
            else a[i] = gelu_tanhf(a[i]) * b[i];
        }
        store4(act + (size_t)t * lda + (f - split / 2u), a);
    }
};
template <typename AT>
struct EpiConvert {
    static constexpr bool kPaired = false, kTrans = false;
    AT* out;
    uint32_t ldo;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f) const { store4(out + (size_t)t * ldo + f, a); }
};
template <typename AT>
struct EpiTransposed {  // f: this lane's feature, t: the first of its four tokens
    static constexpr bool kPaired = false, kTrans = true;
    AT* out;
    uint32_t ldo;
    __device__ void operator()(uint32_t, uint32_t f, uint32_t t, v4f a, v4f) const { store4(out + (size_t)f * ldo + t, a); }
};
struct EpiGates {
    static constexpr bool kPaired = true, kTrans = false;
    GateArgs g;
    uint32_t block;
    __device__ void operator()(uint32_t z, uint32_t f, uint32_t t, v4f r, v4f i) const {
        const uint32_t ch = z * block + f;
        const size_t at = (size_t)t * g.channels + ch;
        r += *reinterpret_cast<const v4f*>(g.r_bias + ch), i += *reinterpret_cast<const v4f*>(g.i_bias + ch);
        const v4f rate = *reinterpret_cast<const v4f*>(g.rate + ch), u = *reinterpret_cast<const v4f*>(g.u + at);
        v4f a, b;
#pragma unroll
        for (int k = 0; k < 4; k++) {
            const float log_a = sigmoidf(r[k]) * rate[k];
            a[k] = expf(log_a);
            b[k] = sqrtf(-expm1f(2.0f * log_a)) * (sigmoidf(i[k]) * u[k]);
        }
        store4(g.a + at, a), store4(g.b + at, b);
    }
};

struct GemmArgs {
    const uint16_t* w;
    size_t w_stride;     // elements between groups / blocks
    uint32_t ldw, mp;
    const void* x;
    uint32_t ldx, n, k, x_stride_z;
    Grouping g;
};

// The workgroup's tile: which weights, which token rows.  false: nothing to do (a grouped launch is sized for the worst case).
struct TileAt {
    uint32_t m0, t0, rows, z;   // first feature, first output row, rows present, block
    const uint16_t* w;
};
__device__ __forceinline__ bool tile_at(const GemmArgs& a, uint32_t bm, uint32_t bn, uint32_t bid, uint32_t count, TileAt& o) {
    // consecutive workgroups go to the eight XCDs in turn: give every XCD a contiguous run of tiles
    if (count % 8u == 0) bid = (bid & 7u) * (count >> 3) + (bid >> 3);
    const uint32_t mtiles = (a.mp + bm - 1) / bm;
    const uint32_t nt = bid / mtiles;
    o.m0 = (bid % mtiles) * bm, o.z = blockIdx.z;
    o.w = a.w + (size_t)blockIdx.z * a.w_stride;
    if (a.g.tiles) {
        if (nt >= *a.g.n_tiles) return false;
        const GroupTile t = a.g.tiles[nt];
        o.w = a.w + (size_t)t.group * a.w_stride;
        o.t0 = t.first, o.rows = t.count;
    } else {
        o.t0 = nt * bn;
        o.rows = a.n - o.t0 < bn ? a.n - o.t0 : bn;
    }
    return true;
}
__device__ __forceinline__ uint32_t source_row(const GemmArgs& a, const TileAt& o, uint32_t r) {
    const uint32_t e = o.t0 + (r < o.rows ? r : o.rows - 1u);  // rows past the end repeat the last one and are not stored
    return a.g.gather ? a.g.gather[e] : e;
}

template <int MT, int NT, class Epi>
__device__ __forceinline__ void run_epilogue(const GemmArgs& a, const TileAt& o, const Epi& epi, const v4f (&acc)[MT][NT], uint32_t wm, uint32_t wn,
                                             uint32_t l16, uint32_t g) {
    if constexpr (Epi::kTrans) {
#pragma unroll
        for (int i = 0; i < MT; i++)
#pragma unroll
            for (int j = 0; j < NT; j++) {
                const uint32_t f = o.m0 + wm + 16 * i + l16, r = wn + 16 * j + 4 * g;
                if (f < a.mp && r < o.rows) epi(o.z, f, o.t0 + r, acc[i][j], acc[i][j]);  // tokens past the end land in the row's padding
            }
    } else {
#pragma unroll
        for (int j = 0; j < NT; j++) {
            const uint32_t r = wn + 16 * j + l16;
            if (r >= o.rows) continue;
            if constexpr (Epi::kPaired) {
#pragma unroll
                for (int i = 0; i < MT; i += 2) {
                    const uint32_t row = o.m0 + wm + 16 * i;  // a multiple of 32
                    if (row < a.mp) epi(o.z, (row >> 1) + 4 * g, o.t0 + r, acc[i][j], acc[i + 1][j]);
                }
            } else {
#pragma unroll
                for (int i = 0; i < MT; i++) {
                    const uint32_t f = o.m0 + wm + 16 * i + 4 * g;
                    if (f < a.mp) epi(o.z, f, o.t0 + r, acc[i][j], acc[i][j]);
                }
            }
        }
    }
}

// Tile `bid` of `count`.
template <int MT, int NT, int PD, int WM, int WN, class Epi>
__device__ __forceinline__ void gemm_bf16_tile(const GemmArgs& a, const Epi& epi, uint32_t bid, uint32_t count) {
    constexpr uint32_t BM = 16 * MT * WM, BN = 16 * NT * WN, BK = 64, THREADS = 64 * WM * WN;
    constexpr int LA = BM * 8 / THREADS, LB = BN * 8 / THREADS;  // 16-byte chunks per thread and step
    __shared__ __align__(16) uint16_t sa[2][BM * BK], sb[2][BN * BK];
    TileAt o;
    if (!tile_at(a, BM, BN, bid, count, o)) return;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4;
    const uint32_t wm = (wave % WM) * (16 * MT), wn = (wave / WM) * (16 * NT);
    const uint16_t* x = static_cast<const uint16_t*>(a.x) + (size_t)o.z * a.x_stride_z;
    const uint16_t *pa[LA], *pb[LB];
    uint32_t da[LA], db[LB];
#pragma unroll
    for (int i = 0; i < LA; i++) {
        const uint32_t c = tid + THREADS * i, row = c >> 3, ch = c & 7u, m = o.m0 + row < a.mp ? o.m0 + row : a.mp - 1u;
        pa[i] = o.w + (size_t)m * a.ldw + ch * 8;
        da[i] = row * BK + ((ch ^ (row & 7u)) << 3);
    }
#pragma unroll
    for (int i = 0; i < LB; i++) {
        const uint32_t c = tid + THREADS * i, row = c >> 3, ch = c & 7u;
        pb[i] = x + (size_t)source_row(a, o, row) * a.ldx + ch * 8;
        db[i] = row * BK + ((ch ^ (row & 7u)) << 3);
    }
    const uint32_t steps = a.k / BK;
    u4 ra[PD][LA], rb[PD][LB];
#pragma unroll
    for (int d = 0; d < PD; d++) {
        const uint32_t k0 = (uint32_t)d < steps ? BK * d : 0u;
#pragma unroll
        for (int i = 0; i < LA; i++) ra[d][i] = *reinterpret_cast<const u4*>(pa[i] + k0);
#pragma unroll
        for (int i = 0; i < LB; i++) rb[d][i] = *reinterpret_cast<const u4*>(pb[i] + k0);
    }
    v4f acc[MT][NT];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < NT; j++) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};
    // Step s + 1 leaves its registers for LDS behind the products of step s, and step s + 1 + PD is requested into them.
    int cur = 0;
    auto advance = [&](u4 (&va)[LA], u4 (&vb)[LB], uint32_t refill, int buf) {
#pragma unroll
        for (int i = 0; i < LA; i++) *reinterpret_cast<u4*>(&sa[buf][da[i]]) = va[i];
#pragma unroll
        for (int i = 0; i < LB; i++) *reinterpret_cast<u4*>(&sb[buf][db[i]]) = vb[i];
        if (refill >= steps) return;
#pragma unroll
        for (int i = 0; i < LA; i++) va[i] = *reinterpret_cast<const u4*>(pa[i] + refill * BK);
#pragma unroll
        for (int i = 0; i < LB; i++) vb[i] = *reinterpret_cast<const u4*>(pb[i] + refill * BK);
    };
    advance(ra[0], rb[0], PD, 0);
    __syncthreads();
    for (uint32_t s0 = 0; s0 < steps; s0 += PD) {
#pragma unroll
        for (int d = 0; d < PD; d++) {
            const uint32_t step = s0 + d;
            if (step >= steps) break;
#pragma unroll
            for (int s = 0; s < 2; s++) {
                bf8 fa[MT], fb[NT];
                const uint32_t ch = (((4 * s + g) ^ (l16 & 7u)) << 3);
#pragma unroll
                for (int i = 0; i < MT; i++) fa[i] = *reinterpret_cast<const bf8*>(&sa[cur][(wm + 16 * i + l16) * BK + ch]);
#pragma unroll
                for (int j = 0; j < NT; j++) fb[j] = *reinterpret_cast<const bf8*>(&sb[cur][(wn + 16 * j + l16) * BK + ch]);
#pragma unroll
                for (int i = 0; i < MT; i++)
#pragma unroll
                    for (int j = 0; j < NT; j++)
                        acc[i][j] = Epi::kTrans ? __builtin_amdgcn_mfma_f32_16x16x32_bf16(fb[j], fa[i], acc[i][j], 0, 0, 0)
                                                : __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
            }
            if (step + 1 < steps) advance(ra[(d + 1) % PD], rb[(d + 1) % PD], step + 1 + PD, cur ^ 1);
            __syncthreads();
            cur ^= 1;
        }
    }
    run_epilogue<MT, NT>(a, o, epi, acc, wm, wn, l16, g);
}

template <int MT, int NT, int PD, int WM, int WN, class Epi>
__global__ __launch_bounds__(64 * WM * WN) void gemm_bf16_kernel(GemmArgs a, Epi epi) {
    gemm_bf16_tile<MT, NT, PD, WM, WN>(a, epi, blockIdx.x, gridDim.x);
}

struct StoresArgs {
    GemmArgs a[kMaxStores];
    EpiStore e[kMaxStores];
    uint32_t first[kMaxStores + 1], count;  // tiles of product i: first[i] .. first[i + 1] - 1
};
template <int MT, int NT, int PD, int WM, int WN>
__global__ __launch_bounds__(64 * WM * WN) void gemm_bf16_stores_kernel(StoresArgs s) {
    uint32_t i = 0;
    while (i + 1 < s.count && blockIdx.x >= s.first[i + 1]) i++;
    gemm_bf16_tile<MT, NT, PD, WM, WN>(s.a[i], s.e[i], blockIdx.x - s.first[i], s.first[i + 1] - s.first[i]);
}

template <class Epi>
__global__ __launch_bounds__(256) void gemm_f32_kernel(GemmArgs a, Epi epi) {
    constexpr int MT = 2, NT = 2;
    constexpr uint32_t BM = 64, BN = 64, BK = 32, LD = BK + 4;
    __shared__ __align__(16) float sa[BM * LD], sb[BN * LD];
    TileAt o;
    if (!tile_at(a, BM, BN, blockIdx.x, gridDim.x, o)) return;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, l16 = lane & 15u, g = lane >> 4;
    const uint32_t wm = (wave & 1u) * 32u, wn = (wave >> 1) * 32u;
    const float* x = static_cast<const float*>(a.x) + (size_t)o.z * a.x_stride_z;
    const uint32_t arow = tid >> 2, ach = (tid & 3u) * 8u;
    const uint16_t* pa = o.w + (size_t)(o.m0 + arow < a.mp ? o.m0 + arow : a.mp - 1u) * a.ldw + ach;
    const float* pb = x + (size_t)source_row(a, o, arow) * a.ldx + ach;
    v4f acc[MT][NT];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < NT; j++) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};
    for (uint32_t k0 = 0; k0 < a.k; k0 += BK) {
        const uint4 wv = *reinterpret_cast<const uint4*>(pa + k0);
        const v4f b0 = *reinterpret_cast<const v4f*>(pb + k0), b1 = *reinterpret_cast<const v4f*>(pb + k0 + 4);
        __syncthreads();  // the previous step's reads are done
        float* da = &sa[arow * LD + ach];
        const uint32_t wq[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
        for (int i = 0; i < 4; i++) da[2 * i] = __uint_as_float(wq[i] << 16), da[2 * i + 1] = __uint_as_float(wq[i] & 0xffff0000u);
        *reinterpret_cast<v4f*>(&sb[arow * LD + ach]) = b0, *reinterpret_cast<v4f*>(&sb[arow * LD + ach + 4]) = b1;
        __syncthreads();
#pragma unroll
        for (uint32_t kk = 0; kk < BK; kk += 4) {
            float fa[MT], fb[NT];
#pragma unroll
            for (int i = 0; i < MT; i++) fa[i] = sa[(wm + 16 * i + l16) * LD + kk + g];
#pragma unroll
            for (int j = 0; j < NT; j++) fb[j] = sb[(wn + 16 * j + l16) * LD + kk + g];
#pragma unroll
            for (int i = 0; i < MT; i++)
#pragma unroll
                for (int j = 0; j < NT; j++)
                    acc[i][j] = Epi::kTrans ? __builtin_amdgcn_mfma_f32_16x16x4f32(fb[j], fa[i], acc[i][j], 0, 0, 0)
                                            : __builtin_amdgcn_mfma_f32_16x16x4f32(fa[i], fb[j], acc[i][j], 0, 0, 0);
        }
    }
    run_epilogue<MT, NT>(a, o, epi, acc, wm, wn, l16, g);
}

// Host-side shape checks every launch goes through: K in whole steps, vector-aligned rows.
bool shapes_fit(const DenseWeight& w, const GemmIn& in, uint32_t k) {
    return w.d && in.x && w.mp % kDensePad == 0 && k % kDensePad == 0 && w.kp % 8u == 0 && k <= w.kp && in.ldx % 8u == 0 &&
           (reinterpret_cast<uintptr_t>(w.d) | reinterpret_cast<uintptr_t>(in.x)) % 16u == 0;
}

template <class Epi>
hipError_t run_gemm(const DenseWeight& w, const GemmIn& in, const Epi& epi, const Launch& L, const Grouping& g = Grouping(), uint32_t z = 1,
                    uint32_t x_stride_z = 0) {
    if (in.n == 0) return hipSuccess;
    if (!shapes_fit(w, in, w.kp) || (g.tiles && (z != 1 || !g.n_tiles || g.max_tiles == 0))) return hipErrorInvalidValue;
    const GemmArgs a{w.d, w.stride, w.kp, w.mp, in.x, in.ldx, in.n, w.kp, x_stride_z, g};
    auto grid = [&](uint32_t bm, uint32_t bn) {
        const uint32_t mt = (w.mp + bm - 1) / bm, nt = g.tiles ? g.max_tiles : (in.n + bn - 1) / bn;
        return dim3(mt * nt, 1, z);
    };
    if (in.f32) return launch_kernel(L, kFamGemm, gemm_f32_kernel<Epi>, grid(64, 64), dim3(256), a, epi);
    if (g.tiles) return launch_kernel(L, kFamGemm, gemm_bf16_kernel<4, 2, 3, 2, 2, Epi>, grid(128, kGroupTileRows), dim3(256), a, epi);
    // the widest tile that leaves no CU without one (a short K is mostly epilogue: small tiles, more of them)
    const dim3 huge = grid(256, 256), big = grid(128, 128), tall = grid(128, 64);
    if (w.kp > 256u && huge.x * huge.z >= 320u) return launch_kernel(L, kFamGemm, gemm_bf16_kernel<4, 4, 1, 4, 4, Epi>, huge, dim3(1024), a, epi);
    if (w.kp > 256u && big.x * big.z >= 192u) return launch_kernel(L, kFamGemm, gemm_bf16_kernel<4, 4, 2, 2, 2, Epi>, big, dim3(256), a, epi);
    if (w.kp > 256u && tall.x * tall.z >= 192u) return launch_kernel(L, kFamGemm, gemm_bf16_kernel<4, 2, 3, 2, 2, Epi>, tall, dim3(256), a, epi);
    return launch_kernel(L, kFamGemm, gemm_bf16_kernel<2, 2, 4, 2, 2, Epi>, grid(64, 64), dim3(256), a, epi);
}

}  // namespace

hipError_t launch_gemm_store(const DenseWeight& w, const GemmIn& in, float* out, uint32_t ldo, const float* add, const Launch& L, const Grouping& g) {
    if (ldo < w.mp || ldo % 4u) return hipErrorInvalidValue;
    return run_gemm(w, in, EpiStore{out, ldo, add}, L, g);
}

hipError_t launch_gemm_stores(const GemmStore* g, uint32_t count, const Launch& L) {
    if (count == 0 || count > kMaxStores) return hipErrorInvalidValue;
    auto tiles = [&](uint32_t i, uint32_t bm, uint32_t bn) { return (g[i].w.mp + bm - 1) / bm * ((g[i].in.n + bn - 1) / bn); };
    uint32_t tall = 0, longest = 0;
    bool f32 = false;
    for (uint32_t i = 0; i < count; i++) {
        if (g[i].in.n == 0 || g[i].ldo < g[i].w.mp || g[i].ldo % 4u || !shapes_fit(g[i].w, g[i].in, g[i].w.kp)) return hipErrorInvalidValue;
        tall += tiles(i, 128, 64), longest = longest < g[i].w.kp ? g[i].w.kp : longest, f32 = f32 || g[i].in.f32;
    }
    if (f32) {
        for (uint32_t i = 0; i < count; i++) {
            const hipError_t e = launch_gemm_store(g[i].w, g[i].in, g[i].out, g[i].ldo, nullptr, L);
            if (e != hipSuccess) return e;
        }
        return hipSuccess;
    }
    auto go = [&](auto kernel, uint32_t bm, uint32_t bn, uint32_t threads) {
        StoresArgs s{};
        s.count = count;
        bool taken[kMaxStores] = {};
        for (uint32_t k = 0; k < count; k++) {  // the longest first
            uint32_t best = kMaxStores;
            for (uint32_t i = 0; i < count; i++)
                if (!taken[i] && (best == kMaxStores || g[i].w.kp > g[best].w.kp)) best = i;
            taken[best] = true;
            const GemmStore& p = g[best];
            s.a[k] = GemmArgs{p.w.d, p.w.stride, p.w.kp, p.w.mp, p.in.x, p.in.ldx, p.in.n, p.w.kp, 0, Grouping()};
            s.e[k] = EpiStore{p.out, p.ldo, nullptr};
            s.first[k + 1] = s.first[k] + tiles(best, bm, bn);
        }
        return launch_kernel(L, kFamGemm, kernel, dim3(s.first[count]), dim3(threads), s);
    };
    if (longest > 256u && tall >= 192u) return go(gemm_bf16_stores_kernel<2, 2, 1, 4, 2>, 128, 64, 512);
    return go(gemm_bf16_stores_kernel<2, 2, 4, 2, 2>, 64, 64, 256);
}

hipError_t launch_gemm_gelu_split(const DenseWeight& w, const GemmIn& in, float* out, uint32_t ldo, const float* bias, uint32_t split, const Launch& L) {
    if (ldo < w.mp || ldo % 4u || split % 4u) return hipErrorInvalidValue;
    return run_gemm(w, in, EpiGeluSplit{out, ldo, bias, split}, L);
}

hipError_t launch_gemm_relu2(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, const Launch& L) {
    if (ldo < w.mp || ldo % 8u) return hipErrorInvalidValue;
    return in.f32 ? run_gemm(w, in, EpiRelu2<float>{static_cast<float*>(out), ldo}, L)
                  : run_gemm(w, in, EpiRelu2<uint16_t>{static_cast<uint16_t*>(out), ldo}, L);
}

hipError_t launch_gemm_silu(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, const float* row_scale, const Launch& L, const Grouping& g) {
    if (ldo < w.mp / 2u || ldo % 8u) return hipErrorInvalidValue;
    return in.f32 ? run_gemm(w, in, EpiSilu<float>{static_cast<float*>(out), ldo, row_scale}, L, g)
                  : run_gemm(w, in, EpiSilu<uint16_t>{static_cast<uint16_t*>(out), ldo, row_scale}, L, g);
}

hipError_t launch_gemm_project(const DenseWeight& w, const GemmIn& in, uint32_t split, float* out, uint32_t ldo, void* act, uint32_t lda, const Launch& L) {
    if (split % kDensePad || split > w.mp || ldo < split || ldo % 4u || (split < w.mp && (!act || lda < (w.mp - split) / 2u || lda % 8u))) return hipErrorInvalidValue;
    return in.f32 ? run_gemm(w, in, EpiProject<float>{out, ldo, split, static_cast<float*>(act), lda}, L)
                  : run_gemm(w, in, EpiProject<uint16_t>{out, ldo, split, static_cast<uint16_t*>(act), lda}, L);
}

hipError_t launch_gemm_convert(const DenseWeight& w, const GemmIn& in, void* out, uint32_t ldo, bool transposed, const Launch& L) {
    if (in.f32 || ldo % 8u || ldo < (transposed ? pad_to(in.n, 4) : w.mp)) return hipErrorInvalidValue;
    uint16_t* o = static_cast<uint16_t*>(out);
    return transposed ? run_gemm(w, in, EpiTransposed<uint16_t>{o, ldo}, L) : run_gemm(w, in, EpiConvert<uint16_t>{o, ldo}, L);
}

hipError_t launch_gemm_gates(const DenseWeight& w, const GemmIn& in, uint32_t blocks, uint32_t x_block_stride, const GateArgs& g, const Launch& L) {
    if (blocks == 0 || w.mp / 2u * blocks != g.channels || x_block_stride % 8u || x_block_stride < w.kp) return hipErrorInvalidValue;
    return run_gemm(w, in, EpiGates{g, w.mp / 2u}, L, Grouping(), blocks, x_block_stride);
}

}  // namespace wick_rocm
