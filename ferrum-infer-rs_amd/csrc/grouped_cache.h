// Layout of the grouped attention's value cache: what its kernels share (layer_ops.h describes both caches).
#pragma once
#include "tiled_gemm.h"

namespace fh {

// place of (token slot, dimension) within a block's values of one head
__device__ __forceinline__ int value_offset(int slot, int d) { return ((((d >> 5) * 4 + (slot >> 2)) * 16 + (d & 15)) * 2 + ((d >> 4) & 1)) * 4 + (slot & 3); }
// Vᵀ operand of 16 dims (half `sub` of a 32-dim load) over the keys of two blocks
__device__ __forceinline__ bf16x8 value_operand(bf16x8 v0, bf16x8 v1, int sub) {
    return sub ? (bf16x8){v0[4], v0[5], v0[6], v0[7], v1[4], v1[5], v1[6], v1[7]} : (bf16x8){v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
}

}  // namespace fh
