// qm_decoder_mfma32.h — fp32 matrix-core products (v_mfma_f32_16x16x4_f32) of the chunked recurrences.
//
// A lane l of group g = l / 16 holds, of a 16 x 16 result, column l % 16 and rows 4 g + r (r = 0..3).  One instruction adds
// four terms of the reduction, group g supplying one of them for both operands; which four is free as long as both operands
// agree.  Here instruction t of a block of 16 takes term 4 g + t: an operand whose reduction runs along memory is then one
// float4 per lane for four instructions, and a result in registers is at once the right operand of a product over its rows.
#pragma once

#include "qm_decoder_device.h"

namespace qm {

__device__ __forceinline__ f32x4_t mfma32(float a, float b, f32x4_t acc) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, acc, 0, 0, 0); }
// acc[16 rows][16 columns] += sum over 16 terms: a = the lane's row, b = the lane's column, terms 4 g .. 4 g + 3
__device__ __forceinline__ f32x4_t mfma32_block(float4 a, float4 b, f32x4_t acc) {
    acc = mfma32(a.x, b.x, acc);
    acc = mfma32(a.y, b.y, acc);
    acc = mfma32(a.z, b.z, acc);
    return mfma32(a.w, b.w, acc);
}
// LDS rows whose float4s, read by sixteen lanes from sixteen rows, lie in different banks
__host__ __device__ inline int mfma32_stride(int columns) { return (columns + 63) / 64 * 64 + 4; }
__host__ __device__ inline int mfma32_pad(int n) { return (n + 15) / 16 * 16; }

}  // namespace qm
