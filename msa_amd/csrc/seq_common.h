// Helpers shared by the recurrent / latent-attention layer kernels (msa_seq.h).
#pragma once

#include <initializer_list>

#include "../../include/msa_seq.h"
#include "common.h"

template <typename T>
__device__ __forceinline__ float to_f32(T v);
template <>
__device__ __forceinline__ float to_f32<bf16_t>(bf16_t v) { return bf16_to_f32(v); }
template <>
__device__ __forceinline__ float to_f32<float>(float v) { return v; }
template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) { return f32_to_bf16(v); }
template <>
__device__ __forceinline__ float from_f32<float>(float v) { return v; }

// fp32 exponential and its relatives on the hardware's 2^x and 1/x (one unit in the last place each).
__device__ __forceinline__ float exp_f(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid_f(float x) { return __builtin_amdgcn_rcpf(1.0f + exp_f(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
__device__ __forceinline__ float softplus_f(float x) { return x > 30.f ? x : log1pf(expf(x)); }
// tanh: its Taylor series where (1 - e) / (1 + e) would cancel, otherwise that.
__device__ __forceinline__ float tanh_f(float x) {
  const float e = exp_f(-2.0f * fabsf(x)), s = x * x;
  const float big = copysignf((1.0f - e) * __builtin_amdgcn_rcpf(1.0f + e), x);
  const float small = x * (1.0f + s * (-0.33333333f + s * (0.13333333f + s * (-0.053968254f + s * 0.021869488f))));
  return fabsf(x) < 0.15f ? small : big;
}
// z (1 + tanh(y)) / 2 = z / (1 + exp(-2 y)), y = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh_f(float z) { return z * sigmoid_f(1.5957691216057308f * (z + 0.044715f * z * z * z)); }

// g sigmoid(alpha g) (u + shift) of a gate and an up projection, clamped from above and on both sides
__device__ __forceinline__ float clamped_glu_f(float gate, float up, float limit, float alpha, float shift) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g * sigmoid_f(alpha * g) * (u + shift);
}

// VEC consecutive elements of a row (aligned to their size, at most 16 bytes), as fp32.
template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 8 && sizeof(T) == 2) {
    const uint4 w = *reinterpret_cast<const uint4*>(p);
    v[0] = bf16lo(w.x); v[1] = bf16hi(w.x); v[2] = bf16lo(w.y); v[3] = bf16hi(w.y);
    v[4] = bf16lo(w.z); v[5] = bf16hi(w.z); v[6] = bf16lo(w.w); v[7] = bf16hi(w.w);
  } else if constexpr (VEC == 8) {
    const float4 w = *reinterpret_cast<const float4*>(p), u = *reinterpret_cast<const float4*>(p + 4);
    v[0] = w.x; v[1] = w.y; v[2] = w.z; v[3] = w.w; v[4] = u.x; v[5] = u.y; v[6] = u.z; v[7] = u.w;
  } else if constexpr (VEC == 2 && sizeof(T) == 2) {
    const uint32_t w = *reinterpret_cast<const uint32_t*>(p);
    v[0] = bf16lo(w); v[1] = bf16hi(w);
  } else if constexpr (VEC == 2) {
    const float2 w = *reinterpret_cast<const float2*>(p);
    v[0] = w.x; v[1] = w.y;
  } else if constexpr (VEC == 4 && sizeof(T) == 2) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    v[0] = bf16lo(w.x); v[1] = bf16hi(w.x); v[2] = bf16lo(w.y); v[3] = bf16hi(w.y);
  } else if constexpr (VEC == 4) {
    const float4 w = *reinterpret_cast<const float4*>(p);
    v[0] = w.x; v[1] = w.y; v[2] = w.z; v[3] = w.w;
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = to_f32<T>(p[i]);
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 8 && sizeof(T) == 2) {
    *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
  } else if constexpr (VEC == 8) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
  } else if constexpr (VEC == 2 && sizeof(T) == 2) {
    *reinterpret_cast<uint32_t*>(p) = pack_bf16x2(v[0], v[1]);
  } else if constexpr (VEC == 2) {
    *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]);
  } else if constexpr (VEC == 4 && sizeof(T) == 2) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  } else if constexpr (VEC == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = from_f32<T>(v[i]);
  }
}

// Host side: vectors are usable when every given address is 16-byte aligned and every stride a multiple of `n` elements.
static inline bool vec_ok(int n, std::initializer_list<const void*> ps, std::initializer_list<int64_t> strides) {
  for (const void* p : ps)
    if (((uintptr_t)p & 15) != 0) return false;
  for (int64_t s : strides)
    if (s % n != 0) return false;
  return true;
}

#define MSA_CHECK_BATCH(b, who)                                                                                     \
  MSA_REQUIRE((b) && (b)->cu && (b)->row_seq && (b)->slot && (b)->pos && (b)->n_seq > 0 && (b)->rows >= (b)->n_seq && \
                  (b)->max_rows > 0 && (b)->max_rows <= (b)->rows && (b)->rows < (1 << 24),                         \
              "%s: bad batch", who)
#define MSA_CHECK_DTYPE(d, who) MSA_REQUIRE((d) == MSA_BF16 || (d) == MSA_F32, "%s: bad dtype %d", who, d)
