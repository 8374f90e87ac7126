// Matrix-core helpers: 16x16x32 bf16 products and transposed LDS reads.
#pragma once
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(4))) unsigned u32x4;

__device__ __forceinline__ f32x4 mfma(u32x4 a, u32x4 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(
      __builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0,
      0);
}

// An operand whose 8 elements lie in 8 successive LDS rows: 16 lanes
// address a 4 x 16 block (lane i: row i / 4, columns 4 (i % 4) ..) and
// each gets one of its columns; the second block is ``down`` further.
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
__device__ __forceinline__ u32x4 load_columns(const unsigned short* p,
                                              int down) {
  const uint2 a = __builtin_bit_cast(
      uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)p));
  const uint2 b = __builtin_bit_cast(
      uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p + down)));
  return u32x4{a.x, a.y, b.x, b.y};
}

typedef __attribute__((ext_vector_type(2))) float f32x2;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
// two floats to bf16, nearest even
__device__ __forceinline__ unsigned to_bf16x2(float lo, float hi) {
  const f32x2 v = {lo, hi};
  return __builtin_bit_cast(unsigned, __builtin_convertvector(v, bf16x2));
}

#define LOG2E 1.4426950408889634f
