// Element access shared by the row-wise kernels of the mixer groups.  Storage
// dtype S is bf16 (raw u16) or fp32.
#pragma once
#include "common.h"

namespace {

template <typename S> __device__ __forceinline__ float ldf(const S* p);
template <> __device__ __forceinline__ float ldf<u16>(const u16* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <typename S> __device__ __forceinline__ void stf(S* p, float v);
template <> __device__ __forceinline__ void stf<u16>(u16* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }

// V = 4: one 8- or 16-byte access (aligned rows); V = 1: one element
template <typename S, int V>
__device__ __forceinline__ void ldv(const S* p, float (&o)[4]) {
  if constexpr (V == 4) {
    if constexpr (sizeof(S) == 2) {
      const s16x4 v = *reinterpret_cast<const s16x4*>(p);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = bf2f((u16)v[j]);
    } else {
      const f32x4 v = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = v[j];
    }
  } else {
    o[0] = ldf<S>(p);
    o[1] = o[2] = o[3] = 0.f;
  }
}
template <typename S, int V>
__device__ __forceinline__ void stv(S* p, const float (&o)[4]) {
  if constexpr (V == 4) {
    if constexpr (sizeof(S) == 2) {
      s16x4 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = (short)f2bf(o[j]);
      *reinterpret_cast<s16x4*>(p) = v;
    } else {
      *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
    }
  } else {
    stf<S>(p, o[0]);
  }
}

// 2 consecutive elements (V2) or one
template <typename S, bool V2>
__device__ __forceinline__ void ld2(const S* p, float& a, float& b) {
  if constexpr (!V2) { a = ldf<S>(p); b = 0.f; }
  else if constexpr (sizeof(S) == 2) {
    const uint32_t w = *reinterpret_cast<const uint32_t*>(p);
    a = bf2f((u16)(w & 0xffffu));
    b = bf2f((u16)(w >> 16));
  } else {
    const f32x2 w = *reinterpret_cast<const f32x2*>(p);
    a = w[0];
    b = w[1];
  }
}
template <typename S, bool V2>
__device__ __forceinline__ void st2(S* p, float a, float b) {
  if constexpr (!V2) stf<S>(p, a);
  else if constexpr (sizeof(S) == 2)
    *reinterpret_cast<uint32_t*>(p) = (uint32_t)f2bf(a) | ((uint32_t)f2bf(b) << 16);
  else *reinterpret_cast<f32x2*>(p) = f32x2{a, b};
}

// tanh-GELU; bf16 storage: tanh from the hardware exponential and reciprocal
// (the result is rounded to 8 bits of mantissa), fp32 storage: the library's
template <typename S> __device__ __forceinline__ float gelu_tanh(float a) {
  const float t = 0.7978845608028654f * (a + 0.044715f * a * a * a);
  if constexpr (sizeof(S) == 2)
    return a - a * __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * t));
  else
    return 0.5f * a * (1.0f + tanhf(t));
}

template <typename... P>
inline bool aligned16(P... p) {
  return ((((uintptr_t)p) % 16 == 0) && ...);
}

inline int grid_for(i64 n) {
  i64 g = (n + 255) / 256;
  return (int)(g < 1 ? 1 : (g > 8192 ? 8192 : g));
}

}  // namespace

#define MIX_DISPATCH(dt, CALL_BF, CALL_F32) \
  do {                                      \
    if ((dt) == 0) { CALL_BF; }             \
    else if ((dt) == 1) { CALL_F32; }       \
    else return 9002;                       \
  } while (0)
