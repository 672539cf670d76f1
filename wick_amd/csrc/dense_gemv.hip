// Matrix-vector products of one token over bfloat16 weights with f32 activations: every product and sum in f32, the weights widened
// exactly.  What comes in front of the product runs in every workgroup's prologue (a few KB out of the L2 each, instead of a launch
// of its own): the residual update with the norm behind the previous sublayer, the norm in front of this one, the input convolution,
// the loop's entry.  The first workgroup also keeps what later launches need: the new residual row and the convolution's newest input.
//
// A wave takes R output rows; its first weight loads are issued before the prologue, whose latency they share.
#include "wick_rocm_dense.h"
#include "wick_rocm_device.h"

namespace wick_rocm {

namespace {

typedef float v4f __attribute__((ext_vector_type(4)));

constexpr uint32_t kThreads = 256;
constexpr uint32_t kGemvMaxK = 15360;  // floats of LDS for the vector

__device__ __forceinline__ float gelu_tanhf(float z) {
    const float s = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * s));
}
__device__ __forceinline__ float siluf(float z) { return z / (1.0f + expf(-z)); }

__device__ __forceinline__ float dot8(uint4 w, float4 a, float4 b, float acc) {
    acc = fmaf(__uint_as_float(w.x << 16), a.x, acc);
    acc = fmaf(__uint_as_float(w.x & 0xffff0000u), a.y, acc);
    acc = fmaf(__uint_as_float(w.y << 16), a.z, acc);
    acc = fmaf(__uint_as_float(w.y & 0xffff0000u), a.w, acc);
    acc = fmaf(__uint_as_float(w.z << 16), b.x, acc);
    acc = fmaf(__uint_as_float(w.z & 0xffff0000u), b.y, acc);
    acc = fmaf(__uint_as_float(w.w << 16), b.z, acc);
    return fmaf(__uint_as_float(w.w & 0xffff0000u), b.w, acc);
}

__device__ __forceinline__ float dot4(v4f a, v4f b) { return (a[0] * b[0] + a[1] * b[1]) + (a[2] * b[2] + a[3] * b[3]); }

__device__ __forceinline__ float block_sum_f32(float v, float* slots) {
    v = wave_sum_f32(v);
    __syncthreads();  // slots may still be read from an earlier call
    if ((threadIdx.x & 63u) == 0) slots[threadIdx.x >> 6] = v;
    __syncthreads();
    return (slots[0] + slots[1]) + (slots[2] + slots[3]);
}

// Two sums in one exchange; slots: eight floats.
__device__ __forceinline__ void block_sum2_f32(float& a, float& b, float* slots) {
    a = wave_sum_f32(a), b = wave_sum_f32(b);
    __syncthreads();
    if ((threadIdx.x & 63u) == 0) slots[threadIdx.x >> 6] = a, slots[4 + (threadIdx.x >> 6)] = b;
    __syncthreads();
    a = (slots[0] + slots[1]) + (slots[2] + slots[3]), b = (slots[4] + slots[5]) + (slots[6] + slots[7]);
}

// Four floats at e of a row that ends at dim (zeros behind it); rows that end at a multiple of four are read as vectors.
__device__ __forceinline__ v4f load_to(const float* p, uint32_t e, uint32_t dim) {
    if (dim % 4u == 0) return *reinterpret_cast<const v4f*>(p + e);
    v4f v;
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = e + i < dim ? p[e + i] : 0.0f;
    return v;
}

enum { kProVec = 0, kProRow = 1, kProRowConv = 2, kProLoop = 3, kProGains = 4 };  // kProGains: a row stage with gains per coordinate

// Fills vec[0 .. k): the vector itself, the row stage's h, or [x | 0 | x0 | 0].  All threads call it; it ends with a barrier.
// A thread owns coordinates 4 t .. 4 t + 3 of every 1024: NQ vectors of four (dim <= 1024 NQ; rows are padded to 64).
template <int PRO, int NQ>
__device__ __forceinline__ void fill_vector(const GemvIn& in, uint32_t k, float* vec, float* slots) {
    const uint32_t tid = threadIdx.x;
    if constexpr (PRO == kProVec) {
        for (uint32_t e = 4u * tid; e < k; e += 4u * kThreads) {
            v4f v = {0.f, 0.f, 0.f, 0.f};
            if (e < in.vec_len) v = *reinterpret_cast<const v4f*>(in.vec + e);
            *reinterpret_cast<v4f*>(vec + e) = v;
        }
        __syncthreads();
        return;
    } else if constexpr (PRO == kProGains) {
        const RowStage& s = in.row;
        const v4f zero = {0.f, 0.f, 0.f, 0.f};
        v4f x[NQ], y[NQ], y2[NQ], wn[NQ];
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const uint32_t e = 4u * (tid + kThreads * i);
            const bool on = e < s.dim;
            x[i] = on ? load_to(s.x, e, s.dim) : zero;
            y[i] = on && s.y ? load_to(s.y, e, s.dim) : zero, y2[i] = on && s.y2 ? load_to(s.y2, e, s.dim) : zero;
            wn[i] = on && s.w_pre ? load_to(s.w_pre, e, s.dim) : v4f{1.f, 1.f, 1.f, 1.f};
            if (on && s.add) x[i] += load_to(s.add, e, s.dim);
        }
        if (s.y) {
            v4f wp[NQ], wp2[NQ];
            float ss = 0.0f, ss2 = 0.0f;
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                const uint32_t e = 4u * (tid + kThreads * i);
                wp[i] = e < s.dim && s.w_post ? load_to(s.w_post, e, s.dim) : v4f{1.f, 1.f, 1.f, 1.f};
                wp2[i] = e < s.dim && s.w_post2 ? load_to(s.w_post2, e, s.dim) : v4f{1.f, 1.f, 1.f, 1.f};
                ss += dot4(y[i], y[i]), ss2 += dot4(y2[i], y2[i]);
            }
            block_sum2_f32(ss, ss2, slots);
            const float sy = s.g_post / sqrtf(ss / (float)s.dim + s.eps), sy2 = s.g_post / sqrtf(ss2 / (float)s.dim + s.eps);
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                x[i] += y[i] * wp[i] * sy;
                if (s.y2) x[i] += y2[i] * wp2[i] * sy2;
            }
        }
        float ss = 0.0f;
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const uint32_t e = 4u * (tid + kThreads * i);
            if (s.x_out && blockIdx.x == 0 && e < s.dim) *reinterpret_cast<v4f*>(s.x_out + e) = x[i];
            ss += dot4(x[i], x[i]);
        }
        const float sx = s.g_pre / sqrtf(block_sum_f32(ss, slots) / (float)s.dim + s.eps);
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const uint32_t e = 4u * (tid + kThreads * i);
            if (e < k) *reinterpret_cast<v4f*>(vec + e) = x[i] * wn[i] * sx;
        }
        __syncthreads();
    } else {
        const RowStage& s = in.row;
        const bool first = blockIdx.x == 0;
        const v4f zero = {0.f, 0.f, 0.f, 0.f};
        v4f x[NQ], y[NQ];
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const uint32_t e = 4u * (tid + kThreads * i);
            x[i] = e < s.dim ? *reinterpret_cast<const v4f*>(s.x + e) : zero;
            y[i] = s.y && e < s.dim ? *reinterpret_cast<const v4f*>(s.y + e) : zero;
        }
        // the inputs of the earlier taps and the convolution's weights are requested before the reductions wait
        constexpr int TP = PRO == kProRowConv ? 4 : 1;  // taps kept in registers; more are read when they are used
        v4f past[TP][NQ], cw[TP][NQ];
        uint32_t pos = 0;
        if constexpr (PRO == kProRowConv) {
            pos = *in.d_pos;
#pragma unroll
            for (int j = 0; j < TP; j++)
#pragma unroll
                for (int i = 0; i < NQ; i++) {
                    const uint32_t e = 4u * (tid + kThreads * i);
                    const bool on = j < (int)s.taps && e < s.dim;
                    cw[j][i] = on ? *reinterpret_cast<const v4f*>(s.conv + (size_t)j * s.x_stride + e) : zero;
                    const uint32_t back = s.taps - 1u - (uint32_t)j;  // this tap's distance
                    past[j][i] = on && back > 0 && pos >= back ? *reinterpret_cast<const v4f*>(s.ring + (size_t)((pos - back) % s.taps) * s.x_stride + e) : zero;
                }
        }
#pragma unroll
        for (int i = 0; i < NQ; i++)
#pragma unroll
            for (int c = 0; c < 4; c++)
                if (4u * (tid + kThreads * i) + c >= s.dim) x[i][c] = y[i][c] = 0.0f;
        if (s.y) {
            float ss = 0.0f;
#pragma unroll
            for (int i = 0; i < NQ; i++) ss += dot4(y[i], y[i]);
            const float sy = s.g_post / sqrtf(block_sum_f32(ss, slots) / (float)s.dim + s.eps);
#pragma unroll
            for (int i = 0; i < NQ; i++) x[i] += y[i] * sy;
        }
        if (s.x_out && first) {
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                const uint32_t e = 4u * (tid + kThreads * i);
                if (e < s.dim) *reinterpret_cast<v4f*>(s.x_out + e) = x[i];
            }
        }
        if constexpr (PRO == kProLoop) {
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                const uint32_t e = 4u * (tid + kThreads * i);
                if (e >= in.x0_at) continue;
                v4f v = e < s.dim ? *reinterpret_cast<const v4f*>(in.x0 + e) : zero;
#pragma unroll
                for (int c = 0; c < 4; c++)
                    if (e + c >= s.dim) v[c] = 0.0f;
                *reinterpret_cast<v4f*>(vec + e) = x[i];
                *reinterpret_cast<v4f*>(vec + in.x0_at + e) = v;
            }
        } else {
            float ss = 0.0f;
#pragma unroll
            for (int i = 0; i < NQ; i++) ss += dot4(x[i], x[i]);
            const float sx = s.g_pre / sqrtf(block_sum_f32(ss, slots) / (float)s.dim + s.eps);
#pragma unroll
            for (int i = 0; i < NQ; i++) {
                const uint32_t e = 4u * (tid + kThreads * i);
                if (e >= k) continue;
                v4f h = x[i] * sx;
                if constexpr (PRO == kProRowConv) {
                    if (e < s.dim) {
                        if (first) *reinterpret_cast<v4f*>(s.ring + (size_t)(pos % s.taps) * s.x_stride + e) = h;
                        v4f c = zero;
#pragma unroll
                        for (int j = 0; j < TP; j++)
                            if (j < (int)s.taps) c += cw[j][i] * (j + 1 == (int)s.taps ? h : past[j][i]);
                        for (uint32_t j = TP; j < s.taps; j++) {
                            const uint32_t back = s.taps - 1u - j;
                            const v4f v = back == 0 ? h : pos >= back ? *reinterpret_cast<const v4f*>(s.ring + (size_t)((pos - back) % s.taps) * s.x_stride + e) : zero;
                            c += *reinterpret_cast<const v4f*>(s.conv + (size_t)j * s.x_stride + e) * v;
                        }
                        h += c;  // (zero past dim: so are the inputs there and the weights)
                    }
                }
                *reinterpret_cast<v4f*>(vec + e) = h;
            }
        }
        __syncthreads();
    }
}

__device__ __forceinline__ uint4 stream_load(const uint16_t* p) {
    typedef uint32_t u4 __attribute__((ext_vector_type(4)));
    const u4 v = __builtin_nontemporal_load(reinterpret_cast<const u4*>(p));
    return uint4{v[0], v[1], v[2], v[3]};
}

// Weight pieces of N rows that a wave requests before its workgroup's prologue: the first 512 P columns.
template <int N, int P = 2>
struct Ahead {
    uint4 w[N][P];
    __device__ __forceinline__ void load(const uint16_t* const (&rows)[N], uint32_t k) {
        const uint32_t at = 8u * (threadIdx.x & 63u);
#pragma unroll
        for (int c = 0; c < P; c++)
#pragma unroll
            for (int r = 0; r < N; r++) w[r][c] = at + 512u * c < k ? stream_load(rows[r] + at + 512u * c) : uint4{0, 0, 0, 0};
    }
};

// acc[r] += this lane's share of rows[r] . vec over [0, k); the first columns are in `a` already.
template <int N, int P>
__device__ __forceinline__ void dot_rows(const uint16_t* const (&rows)[N], const Ahead<N, P>& a, const float* vec, uint32_t k, float (&acc)[N]) {
    uint32_t at = 8u * (threadIdx.x & 63u);
    {
#pragma unroll
        for (int c = 0; c < P; c++) {
            if (at < k) {
                const float4 v0 = *reinterpret_cast<const float4*>(vec + at), v1 = *reinterpret_cast<const float4*>(vec + at + 4);
#pragma unroll
                for (int r = 0; r < N; r++) acc[r] = dot8(a.w[r][c], v0, v1, acc[r]);
            }
            at += 512u;
        }
    }
#pragma unroll 2
    for (; at < k; at += 512u) {
        uint4 w[N];
#pragma unroll
        for (int r = 0; r < N; r++) w[r] = stream_load(rows[r] + at);
        const float4 v0 = *reinterpret_cast<const float4*>(vec + at), v1 = *reinterpret_cast<const float4*>(vec + at + 4);
#pragma unroll
        for (int r = 0; r < N; r++) acc[r] = dot8(w[r], v0, v1, acc[r]);
    }
}

struct DenseArgs {
    const uint16_t* w;
    uint32_t ldw, m, k;
    GemvIn in;
    float* out;
    const float* bias;
    int act;
    uint32_t split;
};

template <int PRO, int NQ, int R>
__global__ __launch_bounds__(256) void gemv_dense_kernel(DenseArgs a) {
    extern __shared__ __align__(16) float vec[];
    __shared__ float slots[8];
    const uint32_t lane = threadIdx.x & 63u, row0 = (blockIdx.x * 4u + (threadIdx.x >> 6)) * R;
    const uint16_t* rows[R];
#pragma unroll
    for (int r = 0; r < R; r++) rows[r] = a.w + (size_t)(row0 + r < a.m ? row0 + r : a.m - 1u) * a.ldw;
    Ahead<R> ahead;
    ahead.load(rows, a.k);
    fill_vector<PRO, NQ>(a.in, a.k, vec, slots);
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.0f;
    dot_rows(rows, ahead, vec, a.k, acc);
#pragma unroll
    for (int r = 0; r < R; r++) {
        float v = wave_sum_f32(acc[r]);
        const uint32_t row = row0 + r;
        if (lane != 0 || row >= a.m) continue;
        if (a.bias) v += a.bias[row];
        if (a.act == kActGeluSplit && row < a.split) v = gelu_tanhf(v);
        if (a.act == kActRelu2) v = fmaxf(v, 0.0f), v = v * v;
        a.out[row] = v;
    }
}

struct ProjectArgs {
    const uint16_t* w;
    uint32_t ldw, split, total, k;   // rows below split as they are, interleaved pairs up to total
    GemvIn in;
    float *out, *act;
};

// R rows a wave: R consecutive plain ones, or R / 2 pairs.
template <int PRO, int NQ, int R>
__global__ __launch_bounds__(256) void gemv_project_kernel(ProjectArgs a) {
    extern __shared__ __align__(16) float vec[];
    __shared__ float slots[8];
    const uint32_t lane = threadIdx.x & 63u, row0 = (blockIdx.x * 4u + (threadIdx.x >> 6)) * R;
    const bool pairs = row0 >= a.split;
    const uint32_t f0 = (row0 - a.split) / 2u;  // the wave's first pair: R / 2 divides 16
    const uint16_t* rows[R];
#pragma unroll
    for (int r = 0; r < R; r++) {
        const uint32_t f = f0 + r / 2, row = pairs ? a.split + (f >> 4) * 32u + (f & 15u) + 16u * (r & 1) : row0 + r;
        rows[r] = a.w + (size_t)(row < a.total ? row : a.total - 1u) * a.ldw;
    }
    Ahead<R> ahead;
    ahead.load(rows, a.k);
    fill_vector<PRO, NQ>(a.in, a.k, vec, slots);
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.0f;
    dot_rows(rows, ahead, vec, a.k, acc);
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = wave_sum_f32(acc[r]);
    if (lane != 0 || row0 >= a.total) return;
#pragma unroll
    for (int r = 0; r < R; r++) {
        if (!pairs) a.out[row0 + r] = acc[r];
        else if (r % 2 == 0) a.act[f0 + r / 2] = gelu_tanhf(acc[r]) * acc[r + 1];
    }
}

// What an attention step's partials come to, gated, as floats of LDS: a thread takes four coordinates of a head and all its partials
// (behind the active ones lies something older: loaded, not used).
__device__ __forceinline__ void fill_merged(const WindowMerge& m, uint32_t k, float* vec) {
    constexpr uint32_t B = 9;
    const WindowShape& s = m.s;
    const uint32_t stride = s.dvp + 4u, len = s.heads * s.vdim;
    const uint32_t pos = *m.d_pos;
    for (uint32_t e = 4u * threadIdx.x; e < k; e += 4u * kThreads) {
        v4f out = {0.f, 0.f, 0.f, 0.f};
        if (e < len) {
            const uint32_t h = e / s.vdim, d = e % s.vdim;
            const float* parts = m.part + (size_t)h * m.splits * stride;
            const v4f z = *reinterpret_cast<const v4f*>(m.w.p + m.w.g_at + h * s.dvp + d);
            float top = -__builtin_inff(), sum = 0.0f;
            for (uint32_t i0 = 0; i0 < m.splits; i0 += B) {
                v4f v[B];
                float2 ml[B];
#pragma unroll
                for (uint32_t j = 0; j < B; j++) {
                    const float* part = parts + (size_t)(i0 + j < m.splits ? i0 + j : 0u) * stride;
                    ml[j] = *reinterpret_cast<const float2*>(part), v[j] = *reinterpret_cast<const v4f*>(part + 4 + d);
                }
                uint32_t tile0;
                const uint32_t active = s.window_tiles(pos, tile0);
                float now = top;
#pragma unroll
                for (uint32_t j = 0; j < B; j++) {
                    if (i0 + j >= active || i0 + j >= m.splits) ml[j].x = -__builtin_inff();
                    now = fmaxf(now, ml[j].x);
                }
                const float keep = expf(top - now);  // (the first partial is always active)
                out *= keep, sum *= keep, top = now;
#pragma unroll
                for (uint32_t j = 0; j < B; j++) {
                    if (i0 + j >= active || i0 + j >= m.splits) continue;
                    const float w = expf(ml[j].x - now);
                    out += v[j] * w, sum += ml[j].y * w;
                }
            }
#pragma unroll
            for (int i = 0; i < 4; i++) out[i] = out[i] / sum / (1.0f + expf(-z[i]));
        }
        *reinterpret_cast<v4f*>(vec + e) = out;
    }
}

struct SegmentArgs {
    GemvSegment s[kMaxSegments];
    WindowMerge merge;                 // of segment `merged`
    uint32_t merged;
    uint32_t first[kMaxSegments + 1];  // workgroups of segment i: first[i] .. first[i + 1] - 1
    uint32_t count;
};

constexpr int kSegmentAhead = 8;

template <int R>
__global__ __launch_bounds__(256) void gemv_segments_kernel(SegmentArgs a) {
    extern __shared__ __align__(16) float vec[];  // [k] | [parts]
    uint32_t i = 0;
    while (i + 1 < a.count && blockIdx.x >= a.first[i + 1]) i++;
    const GemvSegment& s = a.s[i];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, k = s.w.kp, row0 = ((blockIdx.x - a.first[i]) * 4u + (tid >> 6)) * R;
    const uint16_t* rows[R];
#pragma unroll
    for (int r = 0; r < R; r++) rows[r] = s.w.d + (size_t)(row0 + r < s.m ? row0 + r : s.m - 1u) * k;
    Ahead<R, kSegmentAhead> ahead;
    ahead.load(rows, k);
    if (i == a.merged) {
        fill_merged(a.merge, k, vec);
    } else {
        for (uint32_t e = 4u * tid; e < k; e += 4u * kThreads) {
            v4f v = {0.f, 0.f, 0.f, 0.f};
            if (e < s.vec_len) v = load_to(s.vec, e, s.vec_len);
            *reinterpret_cast<v4f*>(vec + e) = v;
        }
    }
    if (s.norm_w) {
        part_rms(vec, s.vec_len, s.parts, s.eps, vec + k);
        const uint32_t len = s.vec_len / s.parts;
        for (uint32_t e = tid; e < s.vec_len; e += kThreads) vec[e] *= vec[k + e / len] * s.norm_w[e];
    }
    __syncthreads();
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.0f;
    dot_rows(rows, ahead, vec, k, acc);
#pragma unroll
    for (int r = 0; r < R; r++) {
        const float v = wave_sum_f32(acc[r]);
        if (lane == 0 && row0 + r < s.m) s.out[row0 + r] = v;
    }
}

struct RoutedArgs {
    RoutedMlp m;
    GemvIn in;
    const uint32_t* d_token;
    const float* act_in;
    float* out;
    uint32_t k, rows;
};

__device__ __forceinline__ uint32_t routed_expert(const RoutedArgs& a, uint32_t s) { return (uint32_t)a.m.table[(size_t)*a.d_token * a.m.top + s]; }

template <int NQ, int R>
__global__ __launch_bounds__(256) void gemv_routed_up_kernel(RoutedArgs a) {
    extern __shared__ __align__(16) float vec[];
    __shared__ float slots[4];
    const RoutedMlp& m = a.m;
    const uint32_t lane = threadIdx.x & 63u, f0 = (blockIdx.x * 4u + (threadIdx.x >> 6)) * R;
    const uint32_t ff = m.gate_up.mp / 2u, routed = m.top * ff, shared = m.shared_gate_up.d ? m.shared_gate_up.mp / 2u : 0u, total = routed + shared;
    // this wave's R features lie inside one expert: R divides 16, every expert's width is a multiple of 64
    const uint16_t* base = m.gate_up.d;
    uint32_t f = 0, ldw = a.k;
    if (f0 < routed) {
        base = m.gate_up.d + (size_t)routed_expert(a, f0 / ff) * m.gate_up.stride, f = f0 % ff;
    } else if (f0 < total) {
        base = m.shared_gate_up.d, f = f0 - routed;
    } else if (f0 == total && shared) {
        base = m.shared_sg, ldw = 0;  // one row, the same for every r
    }
    const uint16_t* rows[2 * R];
#pragma unroll
    for (int r = 0; r < R; r++) {
        const uint32_t fr = f + r;
        rows[2 * r] = base + (size_t)((fr >> 4) * 32u + (fr & 15u)) * ldw;
        rows[2 * r + 1] = base + (size_t)((fr >> 4) * 32u + 16u + (fr & 15u)) * ldw;
    }
    Ahead<2 * R> ahead;
    ahead.load(rows, a.k);
    fill_vector<kProRow, NQ>(a.in, a.k, vec, slots);
    if (f0 > total || (f0 == total && !shared)) return;
    float acc[2 * R];
#pragma unroll
    for (int r = 0; r < 2 * R; r++) acc[r] = 0.0f;
    dot_rows(rows, ahead, vec, a.k, acc);
    if (f0 == total) {
        const float g = wave_sum_f32(acc[0]);
        if (lane == 0) a.out[total] = 1.0f / (1.0f + expf(-g));
        return;
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
        const float g = wave_sum_f32(acc[2 * r]), u = wave_sum_f32(acc[2 * r + 1]);
        if (lane == 0) a.out[f0 + r] = siluf(g) * u;
    }
}

// The experts' rows and the shared one's are one long row over the concatenated activations.  All pieces a wave needs of it (up to
// kDownAhead of 512 columns) are requested before the activations are scaled into LDS.
constexpr int kDownAhead = 10;

template <int R>
__global__ __launch_bounds__(256) void gemv_routed_down_kernel(RoutedArgs a) {
    extern __shared__ __align__(16) float vec[];
    const RoutedMlp& m = a.m;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, row0 = (blockIdx.x * 4u + (tid >> 6)) * R;
    const uint32_t ff = m.down.kp, routed = m.top * ff, shared = m.shared_down.d ? m.shared_down.kp : 0u, total = routed + shared;
    const int32_t* chosen = m.table + (size_t)*a.d_token * m.top;
    auto piece = [&](uint32_t at, uint32_t r) {  // 8 weights of row r from column `at` (segments are multiples of 64 columns)
        const uint32_t row = row0 + r < a.rows ? row0 + r : a.rows - 1u;
        if (at >= total) return uint4{0, 0, 0, 0};
        const uint16_t* p = at < routed ? m.down.d + (size_t)chosen[at / ff] * m.down.stride + (size_t)row * ff + at % ff
                                        : m.shared_down.d + (size_t)row * shared + (at - routed);
        return *reinterpret_cast<const uint4*>(p);
    };
    uint4 w[kDownAhead][R];
#pragma unroll
    for (int c = 0; c < kDownAhead; c++)
#pragma unroll
        for (int r = 0; r < R; r++) w[c][r] = piece(512u * c + 8u * lane, r);
    const float share = 1.0f / (float)m.top, gate = shared ? a.act_in[total] : 0.0f;
    for (uint32_t e = 4u * tid; e < total; e += 4u * kThreads) {
        const v4f v = *reinterpret_cast<const v4f*>(a.act_in + e);
        *reinterpret_cast<v4f*>(vec + e) = v * (e < routed ? share : gate);
    }
    __syncthreads();
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.0f;
#pragma unroll
    for (int c = 0; c < kDownAhead; c++) {
        const uint32_t at = 512u * c + 8u * lane;
        if (at >= total) break;
        const float4 v0 = *reinterpret_cast<const float4*>(vec + at), v1 = *reinterpret_cast<const float4*>(vec + at + 4);
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = dot8(w[c][r], v0, v1, acc[r]);
    }
    for (uint32_t at = 512u * kDownAhead + 8u * lane; at < total; at += 512u) {
        const float4 v0 = *reinterpret_cast<const float4*>(vec + at), v1 = *reinterpret_cast<const float4*>(vec + at + 4);
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = dot8(piece(at, r), v0, v1, acc[r]);
    }
#pragma unroll
    for (int r = 0; r < R; r++) {
        const float v = wave_sum_f32(acc[r]);
        if (lane == 0 && row0 + r < a.rows) a.out[row0 + r] = v;
    }
}

template <int PRO, int NQ>
hipError_t run_dense(const DenseArgs& a, const Launch& L) {
    const uint32_t lds = a.k * 4u;
    if (a.m <= 1024u) return launch_kernel_lds(L, kFamGemv, gemv_dense_kernel<PRO, NQ, 1>, dim3((a.m + 3u) / 4u), dim3(kThreads), lds, a);
    if (a.m <= 8192u) return launch_kernel_lds(L, kFamGemv, gemv_dense_kernel<PRO, NQ, 2>, dim3((a.m + 7u) / 8u), dim3(kThreads), lds, a);
    return launch_kernel_lds(L, kFamGemv, gemv_dense_kernel<PRO, NQ, 4>, dim3((a.m + 15u) / 16u), dim3(kThreads), lds, a);
}

template <int PRO>
hipError_t run_dense_nq(const DenseArgs& a, const Launch& L) {
    const uint32_t dim = a.in.row.dim;
    if (dim <= 1024u) return run_dense<PRO, 1>(a, L);
    if (dim <= 2048u) return run_dense<PRO, 2>(a, L);
    if (dim <= 4096u) return run_dense<PRO, 4>(a, L);
    if (dim <= 8192u) return run_dense<PRO, 8>(a, L);
    return hipErrorInvalidValue;
}

bool row_ok(const RowStage& s, uint32_t k) {
    return s.x && s.dim > 0 && pad_to(s.dim, 4) <= s.x_stride && s.x_stride % 4u == 0 && k <= pad_to(s.dim, kDensePad) * 2u && s.dim <= k && s.x_out != s.x && (!s.conv || (s.ring && s.taps > 0)) && !s.experts;
}

}  // namespace

hipError_t launch_gemv_dense(const DenseWeight& w, uint32_t m, const GemvIn& in, float* out, const float* bias, int act, uint32_t split, const Launch& L) {
    DenseArgs a{w.d, w.kp, m, in.k ? in.k : w.kp, in, out, bias, act, split};
    if (!w.d || !out || m == 0 || m > w.mp || a.k > w.kp || a.k % 8u || a.k > kGemvMaxK || w.kp % 8u) return hipErrorInvalidValue;
    if (in.vec) {
        if (a.in.vec_len == 0) a.in.vec_len = a.k;
        if (a.in.vec_len % 4u) return hipErrorInvalidValue;
        return run_dense<kProVec, 1>(a, L);
    }
    if (!row_ok(in.row, a.k) || (in.row.conv && !in.d_pos)) return hipErrorInvalidValue;
    if (in.x0) {
        if (in.x0_at != pad_to(in.row.dim, kDensePad) || 2u * in.x0_at != a.k) return hipErrorInvalidValue;
        return run_dense_nq<kProLoop>(a, L);
    }
    if (in.row.vector_gains()) return in.row.conv ? hipErrorInvalidValue : run_dense_nq<kProGains>(a, L);
    return in.row.conv ? run_dense_nq<kProRowConv>(a, L) : run_dense_nq<kProRow>(a, L);
}

hipError_t launch_gemv_project(const DenseWeight& w, uint32_t split, const GemvIn& in, float* out, float* act, const Launch& L) {
    const ProjectArgs a{w.d, w.kp, split, w.mp, w.kp, in, out, act};
    if (!w.d || !out || split % kDensePad || split > w.mp || (split < w.mp && !act) || a.k > kGemvMaxK || in.vec || in.x0 || in.row.conv || !row_ok(in.row, a.k))
        return hipErrorInvalidValue;
    constexpr uint32_t R = 4;
    const dim3 grid(w.mp / (4u * R));
    const uint32_t lds = a.k * 4u, dim = in.row.dim;
    if (dim <= 1024u) return launch_kernel_lds(L, kFamGemv, gemv_project_kernel<kProGains, 1, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 2048u) return launch_kernel_lds(L, kFamGemv, gemv_project_kernel<kProGains, 2, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 4096u) return launch_kernel_lds(L, kFamGemv, gemv_project_kernel<kProGains, 4, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 8192u) return launch_kernel_lds(L, kFamGemv, gemv_project_kernel<kProGains, 8, R>, grid, dim3(kThreads), lds, a);
    return hipErrorInvalidValue;
}

hipError_t launch_gemv_segments(const GemvSegment* segs, uint32_t count, const Launch& L) {
    if (count == 0 || count > kMaxSegments) return hipErrorInvalidValue;
    SegmentArgs a{};
    a.count = count, a.merged = kMaxSegments;
    uint32_t lds = 0, rows = 0;
    for (uint32_t i = 0; i < count; i++) rows += segs[i].m;
    const uint32_t R = rows <= 1024u ? 1 : 2;
    for (uint32_t i = 0; i < count; i++) {
        const GemvSegment& s = a.s[i] = segs[i];
        if (s.merge) {
            if (a.merged != kMaxSegments || !window_merge_foldable(*s.merge) || s.merge->s.heads * s.merge->s.vdim > s.w.kp) return hipErrorInvalidValue;
            a.merge = *s.merge, a.merged = i;
        }
        if (!s.w.d || !(s.vec || s.merge) || !s.out || s.m == 0 || s.m > s.w.mp || s.vec_len > s.w.kp || s.w.kp % 8u || s.w.kp > kGemvMaxK || s.parts == 0 || s.vec_len % s.parts ||
            s.parts > 512u)
            return hipErrorInvalidValue;
        a.first[i + 1] = a.first[i] + (s.m + 4u * R - 1u) / (4u * R);
        const uint32_t need = (s.w.kp + s.parts) * 4u;
        lds = need > lds ? need : lds;
    }
    return R == 1 ? launch_kernel_lds(L, kFamGemv, gemv_segments_kernel<1>, dim3(a.first[count]), dim3(kThreads), lds, a)
                  : launch_kernel_lds(L, kFamGemv, gemv_segments_kernel<2>, dim3(a.first[count]), dim3(kThreads), lds, a);
}

uint32_t routed_act_floats(const RoutedMlp& m) { return m.top * (m.gate_up.mp / 2u) + (m.shared_gate_up.d ? m.shared_gate_up.mp / 2u : 0u) + 4u; }

hipError_t launch_gemv_routed_up(const RoutedMlp& m, const GemvIn& in, const uint32_t* d_token, float* act, const Launch& L) {
    RoutedArgs a{m, in, d_token, nullptr, act, m.gate_up.kp, 0};
    const bool shared = m.shared_gate_up.d != nullptr;
    if (!m.gate_up.d || !m.table || m.top == 0 || !d_token || !row_ok(in.row, a.k) || in.row.conv || a.k > kGemvMaxK ||
        (shared && (m.shared_gate_up.kp != a.k || !m.shared_sg)))
        return hipErrorInvalidValue;
    constexpr uint32_t R = 2;
    const uint32_t features = routed_act_floats(m) - 4u, waves = features / R + 1u;
    const dim3 grid((waves + 3u) / 4u);
    const uint32_t lds = a.k * 4u, dim = in.row.dim;
    if (dim <= 1024u) return launch_kernel_lds(L, kFamGemv, gemv_routed_up_kernel<1, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 2048u) return launch_kernel_lds(L, kFamGemv, gemv_routed_up_kernel<2, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 4096u) return launch_kernel_lds(L, kFamGemv, gemv_routed_up_kernel<4, R>, grid, dim3(kThreads), lds, a);
    if (dim <= 8192u) return launch_kernel_lds(L, kFamGemv, gemv_routed_up_kernel<8, R>, grid, dim3(kThreads), lds, a);
    return hipErrorInvalidValue;
}

hipError_t launch_gemv_routed_down(const RoutedMlp& m, uint32_t rows, const float* act, const uint32_t* d_token, float* out, const Launch& L) {
    RoutedArgs a{m, GemvIn(), d_token, act, out, 0, rows};
    const uint32_t total = m.top * m.down.kp + (m.shared_down.d ? m.shared_down.kp : 0u);
    if (!m.down.d || rows == 0 || rows > m.down.mp || m.down.kp != m.gate_up.mp / 2u || total > kGemvMaxK || !d_token ||
        (m.shared_down.d && m.shared_down.kp != m.shared_gate_up.mp / 2u))
        return hipErrorInvalidValue;
    if (rows <= 2048u) return launch_kernel_lds(L, kFamGemv, gemv_routed_down_kernel<1>, dim3((rows + 3u) / 4u), dim3(kThreads), total * 4u, a);
    return launch_kernel_lds(L, kFamGemv, gemv_routed_down_kernel<2>, dim3((rows + 7u) / 8u), dim3(kThreads), total * 4u, a);
}

}  // namespace wick_rocm
