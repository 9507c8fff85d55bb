// Optional terms of masked softmax attention, shared by the row kernels and
// the matrix-core prefill kernel.  For query position i and key j of head h:
//
//   s = q.k * scale
//   s <- cap * tanh(s / cap)                    (cap > 0)
//   s <- s - r1[h] * ln(1 + r2[h] * (i - j))    (r1 given)
//   softmax denominator += exp(sink[h])         (sink given: a keyless,
//                                                valueless, unscaled term)
//
// first > 0: the keys j < first stay visible to every later row whatever the
// chunk or window says (at their true positions).
//
// ldv is the row stride of the value pages in elements: dv for pages of
// their own, dk when the values are the leading dv elements of the key rows
// (vc == kc; latent attention keeps one row per token).
//
// vshare > 1: the value pages have G / vshare heads, each serving vshare
// neighbouring key heads (differential attention: the two maps of a K/V head
// have keys of their own over the same values).
//
// gate: one output-gate logit per (row, head) in the storage dtype, row stride
// ldg; a head's output is multiplied by the logit's sigmoid.  ldo is the row
// stride of the output in elements (at least H * dv).
#pragma once
#include "common.h"

struct AttnExtra {
  const float* sink;   // [H] or null
  const float* r1;     // [H] or null
  const float* r2;     // [H] (with r1)
  float cap;           // 0: no soft cap
  i64 ldv;
  int first;           // 0: no always-visible leading keys
  int vshare;          // key heads per value head
  const void* gate;    // [T, H] at stride ldg, or null
  i64 ldg, ldo;
};

template <typename S>
__device__ __forceinline__ float attn_head_gate(const AttnExtra& ex, size_t t, int h) {
  if (!ex.gate) return 1.0f;
  float z;
  if constexpr (sizeof(S) == 2) z = bf2f(static_cast<const u16*>(ex.gate)[t * ex.ldg + h]);
  else z = static_cast<const float*>(ex.gate)[t * ex.ldg + h];
  return 1.0f / (1.0f + expf(-z));
}

// exact forms (fp32 storage and the row kernels)
__device__ __forceinline__ float attn_softcap(float s, float cap) {
  return cap > 0.f ? cap * tanhf(s / cap) : s;
}
__device__ __forceinline__ float attn_dist_bias(float r1, float r2, int dist) {
  return r1 * logf(1.0f + r2 * (float)dist);
}
// hardware-transcendental soft cap for scores that are rounded to bf16
// weights afterwards: tanh(x) = 1 - 2 / (1 + e^(2x))
__device__ __forceinline__ float attn_softcap_fast(float s, float inv_cap, float cap) {
  const float e = __expf(2.0f * s * inv_cap);
  return cap - 2.0f * cap * __builtin_amdgcn_rcpf(1.0f + e);
}
