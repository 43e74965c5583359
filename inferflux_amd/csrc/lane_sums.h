// The sum over a power of two of neighbouring lanes, in every one of them: neighbours within a row of 16 lanes swap through
// the lanes' own data paths (pairs, quads, mirrored halves of 8, mirrored rows of 16: a few cycles each, where a trip through
// the LDS crossbar costs a token's whole arithmetic); wider groups go on by shuffles.  The order of the additions is fixed by
// the lane numbers.
#pragma once
#include "common.h"

#define DPP_OF(v, ctrl) __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), (ctrl), 0xF, 0xF, true))
// f[k] is 1 where the group has more than 2^k lanes and 0 where not: a step the group does not need adds nothing, and the
// walk has no branches for the steps within a row of 16 lanes.
struct LaneSteps { float f[4]; int lanes; };
__device__ __forceinline__ LaneSteps lane_steps(int KS) {
  return LaneSteps{{KS >= 2 ? 1.f : 0.f, KS >= 4 ? 1.f : 0.f, KS >= 8 ? 1.f : 0.f, KS >= 16 ? 1.f : 0.f}, KS};
}
__device__ __forceinline__ float column_sum(float v, const LaneSteps& st) {
  v = fmaf(st.f[0], DPP_OF(v, 0xB1), v);        // quad_perm [1, 0, 3, 2]
  v = fmaf(st.f[1], DPP_OF(v, 0x4E), v);        // quad_perm [2, 3, 0, 1]
  v = fmaf(st.f[2], DPP_OF(v, 0x141), v);       // row_half_mirror
  v = fmaf(st.f[3], DPP_OF(v, 0x140), v);       // row_mirror
  if (st.lanes >= 32) v += __shfl_xor(v, 16, WAVE);
  if (st.lanes >= 64) v += __shfl_xor(v, 32, WAVE);
  return v;
}

// A workgroup's meeting point for what it wrote to LDS: waits for the wave's own LDS operations and for the others, but
// not for loads from memory that are still on their way into registers (the next stage's), as __syncthreads() would.
#define LDS_BARRIER() asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory")
