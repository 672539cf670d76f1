// One token through two mixers of the same projection, side by side in one launch: windowed attention's workgroups first, the state-space
// block's behind them.  Neither reads what the other writes.
#include "ssd_step.h"
#include "window_attend.h"

namespace wick_rocm {

namespace {

template <int HG, int NP, typename CT>
__global__ __launch_bounds__(256) void parallel_step_kernel(AttendArgs a, SsdStepArgs b, uint32_t attend_blocks) {
    extern __shared__ __align__(16) float lds[];
    if (blockIdx.x < attend_blocks) window_attend_block<HG, NP, CT>(a, blockIdx.x % a.splits, blockIdx.x / a.splits, 0, lds);
    else ssd_step_block(b, blockIdx.x - attend_blocks, lds);
}

}  // namespace

hipError_t launch_parallel_step(const WindowShape& s, const WindowProj& w, void* kc, void* vc, float* scratch, float* attended, uint32_t attended_len,
                                const SsdShape& ss, const SsdWeights& sw, const SsdProj& sp, float* ring, float* state, float* out, const uint32_t* d_pos,
                                WindowMerge* merge, const Launch& L) {
    AttendPlan p;
    if (!d_pos || !merge || !plan_attend(s, w, kc, vc, scratch, 1, 0, d_pos, attended, attended_len, attended_len, true, p) || !ssd_shape_ok(ss, sp))
        return hipErrorInvalidValue;
    *merge = p.merge();
    const uint32_t attend_blocks = p.a.splits * p.blocks_y, lds = p.lds > ssd_step_lds(ss) ? p.lds : ssd_step_lds(ss);
    const dim3 grid(attend_blocks + ssd_step_blocks(ss));
    const SsdStepArgs b{ss, sw, sp, ring, state, out, d_pos};
    return attend_sizes(s, 1, [&](auto hg, auto np) {
        constexpr int HG = decltype(hg)::value, NP = decltype(np)::value;
        return s.f32 ? launch_kernel_lds(L, kFamOther, parallel_step_kernel<HG, NP, float>, grid, dim3(256), lds, p.a, b, attend_blocks)
                     : launch_kernel_lds(L, kFamOther, parallel_step_kernel<HG, NP, uint16_t>, grid, dim3(256), lds, p.a, b, attend_blocks);
    });
}

}  // namespace wick_rocm
