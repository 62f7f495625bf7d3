// Matrix-core operand types and LDS helpers of the sequence-layer kernels.
#pragma once

#include "seq_common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4_t;
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float floatx16_t;
typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int u32x2_t __attribute__((ext_vector_type(2)));
typedef short shortx4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) shortx4_t lds_shortx4_t;

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kOutside = 0x40000000;     // a buffer offset past every extent: reads zeros, writes nothing

// Transposing LDS read of 16-bit elements: within each group of 16 lanes, lanes 4 r .. 4 r + 3 name the four 8-byte
// pieces of row r (r = 0..3, 16 elements) and lane j receives element j of rows 0..3.
__device__ __forceinline__ shortx4_t lds_read_tr16(const bf16_t* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_shortx4_t*)(p));
}
__device__ __forceinline__ bf16x8_t join8(shortx4_t lo, shortx4_t hi) {
  return __builtin_bit_cast(bf16x8_t, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}
// Eight rows (two reads of four, `gap` LDS elements apart) of a 16-bit tile, transposed.
__device__ __forceinline__ bf16x8_t read_tr8(const bf16_t* p, int gap) { return join8(lds_read_tr16(p), lds_read_tr16(p + gap)); }

// fp32 values as bf16 operands: high part and what it leaves over.
__device__ __forceinline__ void split8(const float (&v)[8], bf16x8_t& hi, bf16x8_t& lo) {
  uint32_t h[4], l[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack_bf16x2(v[2 * i], v[2 * i + 1]);
    l[i] = pack_bf16x2(v[2 * i] - bf16lo(h[i]), v[2 * i + 1] - bf16hi(h[i]));
  }
  hi = __builtin_bit_cast(bf16x8_t, make_uint4(h[0], h[1], h[2], h[3]));
  lo = __builtin_bit_cast(bf16x8_t, make_uint4(l[0], l[1], l[2], l[3]));
}
