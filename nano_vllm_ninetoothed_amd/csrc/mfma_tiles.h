// MFMA operand helpers shared by the kernels that keep bf16 tiles row-major in LDS.
#pragma once
#include "mixed_types.h"

namespace mops {

typedef short s16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x16 mfma32(bf16x8 a, bf16x8 b, f32x16 c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// Eight consecutive elements of a row: an operand whose k dimension runs along the rows.
__device__ __forceinline__ bf16x8 tile_row(const uint16_t* tile, int pitch, int row, int k0) {
  return __builtin_bit_cast(bf16x8, load16(tile + row * pitch + k0));
}

// ds_read_b64_tr_b16: the sixteen lanes of a group address a block of 4 rows x 16 columns (lane i: row i / 4, columns
// 4 (i % 4) ..) and lane i receives column i of the four rows.
__device__ __forceinline__ s16x4 tile_block_columns(const uint16_t* tile, int pitch, int row0, int col0, int lane) {
  typedef s16x4 __attribute__((address_space(3))) * lds_ptr;
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(tile + (row0 + ((lane & 15) >> 2)) * pitch + col0 + 4 * (lane & 3)));
}
__device__ __forceinline__ s16x8 join(s16x4 lo, s16x4 hi) { return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7); }

// Operand whose k dimension runs over the rows of the tile, for the 32x32 form: lane l gets column col0 + (l & 31) of the
// rows r0 + 0..3 and r1 + 0..3, where r0 and r1 already include the offset of the lane's half.
__device__ __forceinline__ s16x8 tile_columns(const uint16_t* tile, int pitch, int r0, int r1, int col0, int lane) {
  const int c = col0 + 16 * ((lane >> 4) & 1);
  return join(tile_block_columns(tile, pitch, r0, c, lane), tile_block_columns(tile, pitch, r1, c, lane));
}

// Eight consecutive bf16 of a row of `n` elements from offset i on, zeros behind the end.
__device__ __forceinline__ u32x4 load8_guarded(const uint16_t* row, int i, int n, bool aligned) {
  if (aligned && i + 8 <= n) return load16(row + i);
  u32x4 w = {0u, 0u, 0u, 0u};
#pragma unroll
  for (int e = 0; e < 8; ++e)
    if (i + e < n) w[e >> 1] |= (uint32_t)row[i + e] << (16 * (e & 1));
  return w;
}

// value = hi + lo in bf16: what is kept in 32 bits enters a bf16 product as two operands with 16 significant bits together.
__device__ __forceinline__ void split8(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
  u32x4 h, l;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    h[e] = pack_bf16x2(v[2 * e], v[2 * e + 1]);
    l[e] = pack_bf16x2(v[2 * e] - bf16lo_to_f32(h[e]), v[2 * e + 1] - bf16hi_to_f32(h[e]));
  }
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}

}  // namespace mops
