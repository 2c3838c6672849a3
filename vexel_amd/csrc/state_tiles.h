// Operands of matrix products over recurrent states (decay.hip, forget.hip): float32 values as two bfloat16 parts, and columns of tiles
// in LDS.
#pragma once

#include "ragged.h"

namespace vx {

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ void split(float v, bf16 *hi, bf16 *lo) {
    *hi = (bf16)v;
    *lo = (bf16)(v - (float)*hi);
}

// Four rows x 16 columns of 16-bit elements, transposed on the way: of a group of 16 lanes, lane i points at columns 4 (i & 3) ..
// of row i >> 2 and gets column i of the four rows.
__device__ __forceinline__ s16x4 read_transposed(const void *p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4 *)p);
}
// Rows r0 + 8 (lane / 16) .. + 7 of column c0 + lane % 16.
__device__ __forceinline__ bf16x8 column8(const bf16 *tile, int ld, int r0, int c0, int lane) {
    const int i = lane & 15;
    const bf16 *p = tile + (r0 + (lane >> 4) * 8 + (i >> 2)) * ld + c0 + (i & 3) * 4;
    const s16x4 a = read_transposed(p), b = read_transposed(p + 4 * ld);
    return __builtin_bit_cast(bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
}

}  // namespace vx
