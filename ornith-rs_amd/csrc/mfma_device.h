// Operand layouts that the matrix-core kernels of the layer-list designs share.
#pragma once

#include "dmath.h"

// bf16 high part and the rest: a 32-bit number as two operands of the matrix cores
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = dm_f2bf2(a, b);
  lo = dm_f2bf2(a - dm_bf2f_lo(hi), b - dm_bf2f_hi(hi));
}

// position of token j (0..31) of a 32-token group in a row of a turned value tile: the order in which
// the lanes of a transposed score tile hold the tokens
__device__ __forceinline__ int vt_pos(int j) { return 8 * ((j & 15) >> 2) + 4 * (j >> 4) + (j & 3); }

// Where a chunk's state (value x key) lies: bf16 in 16 x 32 pieces of 1 KB laid out as the matrix cores
// read them: value row j, key channel d -> 16-byte piece (j % 16) + 16 (d % 32 / 8), element d % 8.
__device__ __forceinline__ size_t s0_at(int DP, int j, int d) {
  return ((size_t)(j >> 4) * (DP >> 5) + (d >> 5)) * 512 + (size_t)((j & 15) + 16 * ((d & 31) >> 3)) * 8 + (d & 7);
}
