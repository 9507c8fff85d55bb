// Row-wise glue kernels of parallel-residual hybrid decoders: fp32 residual
// stream, zero-centred RMSNorm pairs with token shift, per-head output norm
// with SiLU gate, PolyNorm activation, sigmoid-gated residual add, softcap.
//
// Storage dtype S is bf16 (raw u16) or fp32; every statistic, gate and the
// residual itself are fp32.  One workgroup (256 threads = 4 waves) per row
// unless noted; rows are short (model width), so a row is read once into
// registers/LDS-free strided loops and reduced with 64-wide wave shuffles.
#include "common.h"

namespace {

template <typename S> __device__ __forceinline__ float ldf(const S* p);
template <> __device__ __forceinline__ float ldf<u16>(const u16* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <typename S> __device__ __forceinline__ void stf(S* p, float v);
template <> __device__ __forceinline__ void stf<u16>(u16* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }

// 4 consecutive elements (8 B of bf16 / 16 B of fp32); callers guarantee the
// alignment (row lengths and strides multiples of 4, 16-byte aligned bases).
template <typename S> __device__ __forceinline__ void ld4(const S* p, float (&o)[4]);
template <> __device__ __forceinline__ void ld4<u16>(const u16* p, float (&o)[4]) {
  const s16x4 v = *reinterpret_cast<const s16x4*>(p);
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = bf2f((u16)v[j]);
}
template <> __device__ __forceinline__ void ld4<float>(const float* p, float (&o)[4]) {
  const f32x4 v = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = v[j];
}
template <typename S> __device__ __forceinline__ void st4(S* p, const float (&o)[4]);
template <> __device__ __forceinline__ void st4<u16>(u16* p, const float (&o)[4]) {
  s16x4 v;
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = (short)f2bf(o[j]);
  *reinterpret_cast<s16x4*>(p) = v;
}
template <> __device__ __forceinline__ void st4<float>(float* p, const float (&o)[4]) {
  *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
}
// V = 4: vector accesses; V = 1: scalar fallback for odd sizes.
template <typename S, int V>
__device__ __forceinline__ void ldv(const S* p, float (&o)[4]) {
  if (V == 4) ld4<S>(p, o);
  else { o[0] = ldf<S>(p); o[1] = o[2] = o[3] = 0.f; }
}
template <typename S, int V>
__device__ __forceinline__ void stv(S* p, const float (&o)[4]) {
  if (V == 4) st4<S>(p, o);
  else stf<S>(p, o[0]);
}

// Block-wide sum of up to N values per thread (256 threads); every thread
// gets the totals.  red must hold N*4 floats.
template <int N>
__device__ __forceinline__ void block_sum(float (&v)[N], float* red) {
#pragma unroll
  for (int n = 0; n < N; ++n) v[n] = wave_sum_f32(v[n]);
  const int wave = threadIdx.x >> 6;
  __syncthreads();  // red may still be read from a previous call
  if ((threadIdx.x & 63) == 0) {
#pragma unroll
    for (int n = 0; n < N; ++n) red[n * 4 + wave] = v[n];
  }
  __syncthreads();
#pragma unroll
  for (int n = 0; n < N; ++n)
    v[n] = red[n * 4] + red[n * 4 + 1] + red[n * 4 + 2] + red[n * 4 + 3];
}

template <typename S>
__global__ void __launch_bounds__(256) embed_kernel(
    float* __restrict__ out, const S* __restrict__ table,
    const i32* __restrict__ ids, const float* __restrict__ add, float scale,
    int W) {
  const int t = blockIdx.x;
  const S* src = table + (size_t)ids[t] * W;
  float* dst = out + (size_t)t * W;
  for (int i = threadIdx.x; i < W; i += 256)
    dst[i] = ldf<S>(src + i) * scale + (add ? add[i] : 0.f);
}

// x = table[token] + pairs[row of (previous token, token)]: the pair row is
// (previous * mul_prev + token * mul_cur) mod buckets, row `buckets` where a
// sequence starts.  The token before a chunk comes from the sequence's slot of
// `prev` [slots].  STEP: every chunk is a single row, which leaves its token
// in the slot itself; longer chunks leave it through last_token_kernel.
template <typename S, int V, bool STEP>
__global__ void __launch_bounds__(256) embed_pairs_kernel(
    float* __restrict__ out, const S* __restrict__ table,
    const S* __restrict__ pairs, const i32* __restrict__ ids, i32* prev,
    const i32* __restrict__ row_seq, const i32* __restrict__ cu,
    const i32* __restrict__ q_start, const i32* __restrict__ sslot,
    i64 mul_prev, i64 mul_cur, i64 buckets, int W) {
  const int t = blockIdx.x;
  const int b = row_seq[t];
  const int k = t - cu[b];
  const i64 tok = ids[t];
  i64 row = buckets;
  if (k > 0 || q_start[b] > 0) {
    const i64 before = k > 0 ? ids[t - 1] : prev[sslot[b]];
    row = (before * mul_prev + tok * mul_cur) % buckets;
    if (row < 0) row += buckets;
  }
  if (STEP) {
    __syncthreads();                       // every thread has read the slot
    if (threadIdx.x == 0) prev[sslot[b]] = (i32)tok;
  }
  const S* a = table + (size_t)tok * W;
  const S* p = pairs + (size_t)row * W;
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    float av[4], pv[4];
    ldv<S, V>(a + i, av);
    ldv<S, V>(p + i, pv);
#pragma unroll
    for (int j = 0; j < V; ++j) av[j] += pv[j];
    stv<float, V>(out + (size_t)t * W + i, av);
  }
}

__global__ void __launch_bounds__(256) last_token_kernel(
    i32* __restrict__ prev, const i32* __restrict__ ids,
    const i32* __restrict__ cu, const i32* __restrict__ sslot, int B) {
  const int b = blockIdx.x * 256 + threadIdx.x;
  if (b < B && cu[b + 1] > cu[b]) prev[sslot[b]] = ids[cu[b + 1] - 1];
}

__global__ void __launch_bounds__(256) add_rows_kernel(
    float* __restrict__ x, const float* __restrict__ other,
    const float* __restrict__ vec, i64 n, int W) {
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < n;
       i += (i64)gridDim.x * 256) {
    float v = x[i];
    if (other) v += other[i];
    if (vec) v += vec[i % W];
    x[i] = v;
  }
}

// a = norm(x)(1+w1), b = norm(x)(1+w2), s = a + (a_prev - a)*shift.
template <typename S, int V>
__global__ void __launch_bounds__(256) dual_norm_shift_kernel(
    S* __restrict__ a_out, S* __restrict__ s_out, S* __restrict__ b_out,
    float* __restrict__ last, const float* __restrict__ x,
    const S* __restrict__ w1, const S* __restrict__ w2,
    const S* __restrict__ shift, float* prev,
    const i32* __restrict__ row_seq, const i32* __restrict__ cu,
    const i32* __restrict__ q_start, const i32* __restrict__ sslot,
    float eps, int W) {
  // last == nullptr: every chunk is a single row (a decode step); the row's
  // norm goes straight into its state slot, each element read before it is
  // overwritten by the same thread.
  __shared__ float red[8];
  const int t = blockIdx.x;
  const int b = row_seq[t];
  const int r0 = cu[b];
  const bool first = (t == r0);
  const bool is_last = (t == cu[b + 1] - 1);
  const int pos = q_start[b] + (t - r0);
  const float* xr = x + (size_t)t * W;
  const float* xp = xr - W;  // previous row, only touched when !first
  const bool need_prev_row = shift && !first;
  float ss[2] = {0.f, 0.f};
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    float xv[4], pv4[4];
    ldv<float, V>(xr + i, xv);
#pragma unroll
    for (int j = 0; j < V; ++j) ss[0] += xv[j] * xv[j];
    if (need_prev_row) {
      ldv<float, V>(xp + i, pv4);
#pragma unroll
      for (int j = 0; j < V; ++j) ss[1] += pv4[j] * pv4[j];
    }
  }
  block_sum<2>(ss, red);
  const float r = 1.0f / sqrtf(ss[0] / (float)W + eps);
  const float rp = 1.0f / sqrtf(ss[1] / (float)W + eps);
  const float* pv = (shift && first && pos > 0)
                        ? prev + (size_t)sslot[b] * W : nullptr;
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    float xv[4], g1[4], a[4], o[4], tmp[4];
    ldv<float, V>(xr + i, xv);
    ldv<S, V>(w1 + i, g1);
#pragma unroll
    for (int j = 0; j < V; ++j) { g1[j] += 1.0f; a[j] = xv[j] * r * g1[j]; }
    stv<S, V>(a_out + (size_t)t * W + i, a);
    if (b_out) {
      ldv<S, V>(w2 + i, tmp);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = xv[j] * r * (1.0f + tmp[j]);
      stv<S, V>(b_out + (size_t)t * W + i, o);
    }
    if (shift) {
      float ap[4] = {0.f, 0.f, 0.f, 0.f};
      if (need_prev_row) {
        ldv<float, V>(xp + i, tmp);
#pragma unroll
        for (int j = 0; j < V; ++j) ap[j] = tmp[j] * rp * g1[j];
      } else if (pv) {
        ldv<float, V>(pv + i, ap);
      }
      ldv<S, V>(shift + i, tmp);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = a[j] + (ap[j] - a[j]) * tmp[j];
      stv<S, V>(s_out + (size_t)t * W + i, o);
      if (is_last)
        stv<float, V>(last ? last + (size_t)b * W + i
                           : prev + (size_t)sslot[b] * W + i, a);
    }
  }
}

__global__ void __launch_bounds__(256) scatter_state_kernel(
    float* __restrict__ prev, const float* __restrict__ last,
    const i32* __restrict__ sslot, const i32* __restrict__ cu, int W) {
  const int b = blockIdx.x;
  if (cu[b + 1] == cu[b]) return;
  float* dst = prev + (size_t)sslot[b] * W;
  const float* src = last + (size_t)b * W;
  for (int i = threadIdx.x; i < W; i += 256) dst[i] = src[i];
}

template <typename S>
__global__ void __launch_bounds__(256) norm_rows_kernel(
    S* __restrict__ out, const float* __restrict__ x, const S* __restrict__ w,
    const i32* __restrict__ rows, float eps, int W, int one_plus, int center) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  const float* xr = x + (size_t)(rows ? rows[r] : r) * W;
  float mean = 0.f;
  if (center) {
    float sm[1] = {0.f};
    for (int i = threadIdx.x; i < W; i += 256) sm[0] += xr[i];
    block_sum<1>(sm, red);
    mean = sm[0] / (float)W;
  }
  float ss[1] = {0.f};
  for (int i = threadIdx.x; i < W; i += 256) ss[0] += (xr[i] - mean) * (xr[i] - mean);
  block_sum<1>(ss, red);
  const float rs = 1.0f / sqrtf(ss[0] / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += 256) {
    const float g = ldf<S>(w + i) + (one_plus ? 1.0f : 0.f);
    stf<S>(out + (size_t)r * W + i, (xr[i] - mean) * rs * g);
  }
}

// Layer norms on both sides of a sublayer, in one pass over the row:
//   x += mult * LN(y) * w_post        (y given: the previous sublayer's output)
//   h  = LN(x) * w_pre                (h given: the next sublayer's input)
// LN(u) = (u - mean) / sqrt(mean((u - mean)^2) + eps), the variance taken
// from the deviations in a second sum.  x is the fp32 residual, y in Y.
// REG: the row fits 4 passes of the workgroup and waits in registers between
// the sums; otherwise it is read again (x through memory).
constexpr int SWN_IT = 4;

template <typename S, typename Y, int V, int NT, bool REG>
__global__ void __launch_bounds__(NT) sandwich_norm_kernel(
    float* __restrict__ x, S* __restrict__ h, const Y* __restrict__ y,
    i64 ldy, const S* __restrict__ w_post, const S* __restrict__ w_pre,
    float mult, float eps, int W) {
  __shared__ float red[NT / 64];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * W;
  auto total = [&](float v) {                // fixed order, every thread
    v = wave_sum_f32(v);
    __syncthreads();                         // red may still be read
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NT / 64; ++i) s += red[i];
    return s;
  };
  const float inv_w = 1.0f / (float)W;
  if constexpr (REG) {
    float xv[SWN_IT][4], uv[SWN_IT][4];
    float s = 0.f;
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
        ldv<float, V>(xr + i, xv[p]);
        if (y) {
          ldv<Y, V>(y + (size_t)t * ldy + i, uv[p]);
#pragma unroll
          for (int j = 0; j < V; ++j) s += uv[p][j];
        }
      }
    }
    if (y) {
      const float mean = total(s) * inv_w;
      s = 0.f;
#pragma unroll
      for (int p = 0; p < SWN_IT; ++p) {
        const int i = (p * NT + threadIdx.x) * V;
        if (i < W) {
#pragma unroll
          for (int j = 0; j < V; ++j) {
            uv[p][j] -= mean;
            s += uv[p][j] * uv[p][j];
          }
        }
      }
      const float f = mult / sqrtf(total(s) * inv_w + eps);
#pragma unroll
      for (int p = 0; p < SWN_IT; ++p) {
        const int i = (p * NT + threadIdx.x) * V;
        if (i < W) {
          float wv[4];
          ldv<S, V>(w_post + i, wv);
#pragma unroll
          for (int j = 0; j < V; ++j) xv[p][j] += uv[p][j] * f * wv[j];
          stv<float, V>(xr + i, xv[p]);
        }
      }
    }
    if (!h) return;
    s = 0.f;
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
#pragma unroll
        for (int j = 0; j < V; ++j) s += xv[p][j];
      }
    }
    const float mean = total(s) * inv_w;
    s = 0.f;
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
#pragma unroll
        for (int j = 0; j < V; ++j) {
          xv[p][j] -= mean;
          s += xv[p][j] * xv[p][j];
        }
      }
    }
    const float rs = 1.0f / sqrtf(total(s) * inv_w + eps);
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
        float wv[4];
        ldv<S, V>(w_pre + i, wv);
#pragma unroll
        for (int j = 0; j < V; ++j) wv[j] *= xv[p][j] * rs;
        stv<S, V>(h + (size_t)t * W + i, wv);
      }
    }
  } else {
    float v[4], wv[4], u[4];
    float s = 0.f;
    if (y) {
      const Y* yr = y + (size_t)t * ldy;
      for (int i = threadIdx.x * V; i < W; i += NT * V) {
        ldv<Y, V>(yr + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) s += u[j];
      }
      const float mean = total(s) * inv_w;
      s = 0.f;
      for (int i = threadIdx.x * V; i < W; i += NT * V) {
        ldv<Y, V>(yr + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) s += (u[j] - mean) * (u[j] - mean);
      }
      const float f = mult / sqrtf(total(s) * inv_w + eps);
      for (int i = threadIdx.x * V; i < W; i += NT * V) {
        ldv<Y, V>(yr + i, u);
        ldv<S, V>(w_post + i, wv);
        ldv<float, V>(xr + i, v);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] += (u[j] - mean) * f * wv[j];
        stv<float, V>(xr + i, v);            // read back by the same thread
      }
    }
    if (!h) return;
    s = 0.f;
    for (int i = threadIdx.x * V; i < W; i += NT * V) {
      ldv<float, V>(xr + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) s += v[j];
    }
    const float mean = total(s) * inv_w;
    s = 0.f;
    for (int i = threadIdx.x * V; i < W; i += NT * V) {
      ldv<float, V>(xr + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) s += (v[j] - mean) * (v[j] - mean);
    }
    const float rs = 1.0f / sqrtf(total(s) * inv_w + eps);
    for (int i = threadIdx.x * V; i < W; i += NT * V) {
      ldv<float, V>(xr + i, v);
      ldv<S, V>(w_pre + i, wv);
#pragma unroll
      for (int j = 0; j < V; ++j) wv[j] *= (v[j] - mean) * rs;
      stv<S, V>(h + (size_t)t * W + i, wv);
    }
  }
}

// xIELU: z > 0: cp z^2 + z/2;  z <= 0: cn (e^z - 1 - z) + z/2, with (cp, cn)
// in coef.  bf16 storage takes the hardware exponential.
template <typename S, int V>
__global__ void __launch_bounds__(256) xielu_kernel(
    S* __restrict__ out, const S* __restrict__ z, i64 ldz,
    const float* __restrict__ coef, int T, int F) {
  const float cp = coef[0], cn = coef[1];
  const i64 per = F / V;
  const i64 total = (i64)T * per;
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < total;
       i += (i64)gridDim.x * 256) {
    const i64 t = i / per;
    const int c = (int)(i % per) * V;
    float v[4];
    ldv<S, V>(z + t * ldz + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float a = v[j];
      const float n = fminf(a, 0.f);
      const float e = sizeof(S) == 2 ? __expf(n) - 1.0f : expm1f(n);
      v[j] = (a > 0.f ? cp * a * a : cn * (e - n)) + 0.5f * a;
    }
    stv<S, V>(out + t * F + c, v);
  }
}

// Residual add of a layer whose sublayers share one input, and the RMSNorm in
// front of the next layer, in one pass over the row:
//   u = a + sum_s parts[s] + sum_r wts[r] ys[pos[r]] + (sum_i idw[i]) hin
//   x += mult * u (+ vec);   h = x / sqrt(mean(x^2) + eps) * w
// a: what sits in token order (or null); parts [np, T, W] fp32: the same as
// partial sums of a split product (np 0: none); ys: rows in another order, pos < 0
// skipped (top 0: none); hin: the layer's own input under the weights idw [nid]
// at row stride ldi (nid 0: none); vec: one fp32 row; h null: no norm.
// REG: the row fits 4 passes of the workgroup and waits in registers for the
// sum; otherwise it is read again.
template <typename S, int V, int NT, bool REG>
__global__ void __launch_bounds__(NT) residual_norm_kernel(
    float* __restrict__ x, S* __restrict__ h, const S* __restrict__ a, i64 lda,
    const float* __restrict__ parts, int np, const S* __restrict__ ys,
    const i32* __restrict__ pos, const float* __restrict__ wts, int top,
    const S* __restrict__ hin, const float* __restrict__ idw, i64 ldi, int nid,
    float mult, const float* __restrict__ vec, const S* __restrict__ w,
    float eps, int W) {
  __shared__ float red[NT / 64];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * W;
  float fid = 0.f;
  for (int i = 0; i < nid; ++i) fid += idw[(size_t)t * ldi + i];
  const i32* pr = pos + (size_t)t * top;
  const float* wr = wts + (size_t)t * top;
  auto update = [&](int i, float (&xv)[4]) {
    float u[4] = {0.f, 0.f, 0.f, 0.f}, v[4];
    ldv<float, V>(xr + i, xv);
    if (a) ldv<S, V>(a + (size_t)t * lda + i, u);
#pragma unroll 8
    for (int s = 0; s < np; ++s) {
      ldv<float, V>(parts + ((size_t)s * gridDim.x + t) * W + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += v[j];
    }
    for (int r = 0; r < top; ++r) {
      const int p = pr[r];
      if (p < 0) continue;
      const float f = wr[r];
      ldv<S, V>(ys + (size_t)p * W + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += f * v[j];
    }
    if (fid != 0.f) {
      ldv<S, V>(hin + (size_t)t * W + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += fid * v[j];
    }
#pragma unroll
    for (int j = 0; j < V; ++j) xv[j] += mult * u[j];
    if (vec) {
      ldv<float, V>(vec + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) xv[j] += v[j];
    }
    stv<float, V>(xr + i, xv);
  };
  float xs[SWN_IT][4];
  float ss = 0.f;
  if constexpr (REG) {
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
        update(i, xs[p]);
#pragma unroll
        for (int j = 0; j < V; ++j) ss += xs[p][j] * xs[p][j];
      }
    }
  } else {
    for (int i = threadIdx.x * V; i < W; i += NT * V) {
      update(i, xs[0]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += xs[0][j] * xs[0][j];
    }
  }
  if (!h) return;
  ss = wave_sum_f32(ss);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) ss += red[i];
  const float rs = 1.0f / sqrtf(ss / (float)W + eps);
  float wv[4];
  if constexpr (REG) {
#pragma unroll
    for (int p = 0; p < SWN_IT; ++p) {
      const int i = (p * NT + threadIdx.x) * V;
      if (i < W) {
        ldv<S, V>(w + i, wv);
#pragma unroll
        for (int j = 0; j < V; ++j) wv[j] *= xs[p][j] * rs;
        stv<S, V>(h + (size_t)t * W + i, wv);
      }
    }
  } else {
    for (int i = threadIdx.x * V; i < W; i += NT * V) {
      ldv<float, V>(xr + i, xs[0]);          // written by the same thread
      ldv<S, V>(w + i, wv);
#pragma unroll
      for (int j = 0; j < V; ++j) wv[j] *= xs[0][j] * rs;
      stv<S, V>(h + (size_t)t * W + i, wv);
    }
  }
}

// out = max(z, 0)^2 * f, rows of z at stride ldz, of out at ldo.  f is 1 in the
// first `lead` columns, then rw[t, (c - lead) / unit] (rw null: 1 everywhere).
template <typename S, int V>
__global__ void __launch_bounds__(256) relu2_kernel(
    S* __restrict__ out, i64 ldo, const S* __restrict__ z, i64 ldz,
    const float* __restrict__ rw, i64 ldrw, int lead, int unit, int T, int F) {
  const i64 per = F / V;
  const i64 total = (i64)T * per;
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < total;
       i += (i64)gridDim.x * 256) {
    const i64 t = i / per;
    const int c = (int)(i % per) * V;
    const float f = (rw && c >= lead) ? rw[t * ldrw + (c - lead) / unit] : 1.0f;
    float v[4];
    ldv<S, V>(z + t * ldz + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float r = fmaxf(v[j], 0.f);
      v[j] = r * r * f;
    }
    stv<S, V>(out + t * ldo + c, v);
  }
}

// One wave per (row, head): RMS over dv of fp32 o, * weight, * silu(gate)
// (SIG: * sigmoid(gate)).
template <typename S, int V, bool SIG>
__global__ void __launch_bounds__(256) headnorm_gate_kernel(
    S* __restrict__ out, const float* __restrict__ o, const S* __restrict__ g,
    const S* __restrict__ w, float eps, int n_rh, int H, int dv, i64 ldg) {
  const int rh = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (rh >= n_rh) return;
  const int lane = threadIdx.x & 63;
  const int t = rh / H, h = rh % H;
  const float* orow = o + ((size_t)t * H + h) * dv;
  float ss = 0.f;
  for (int d = lane * V; d < dv; d += 64 * V) {
    float ov[4];
    ldv<float, V>(orow + d, ov);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += ov[j] * ov[j];
  }
  ss = wave_sum_f32(ss);
  const float rs = 1.0f / sqrtf(ss / (float)dv + eps);
  const S* grow = g + (size_t)t * ldg + (size_t)h * dv;
  for (int d = lane * V; d < dv; d += 64 * V) {
    float ov[4], gv[4], wv[4] = {1.f, 1.f, 1.f, 1.f}, r[4];
    ldv<float, V>(orow + d, ov);
    ldv<S, V>(grow + d, gv);
    if (w) ldv<S, V>(w + d, wv);
#pragma unroll
    for (int j = 0; j < V; ++j)
      r[j] = ov[j] * rs * wv[j] * ((SIG ? 1.0f : gv[j]) / (1.0f + expf(-gv[j])));
    stv<S, V>(out + ((size_t)t * H + h) * dv + d, r);
  }
}

template <typename S, int V>
__global__ void __launch_bounds__(256) polynorm_kernel(
    S* __restrict__ out, const S* __restrict__ z, const float* __restrict__ coef,
    float eps, int F, i64 ldz) {
  __shared__ float red[12];
  const int t = blockIdx.x;
  const S* zr = z + (size_t)t * ldz;
  float s[3] = {0.f, 0.f, 0.f};
  for (int i = threadIdx.x * V; i < F; i += 256 * V) {
    float v[4];
    ldv<S, V>(zr + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float v2 = v[j] * v[j];
      s[0] += v2;
      s[1] += v2 * v2;
      s[2] += v2 * v2 * v2;
    }
  }
  block_sum<3>(s, red);
  const float r1 = 1.0f / sqrtf(s[0] / (float)F + eps);
  const float r2 = 1.0f / sqrtf(s[1] / (float)F + eps);
  const float r3 = 1.0f / sqrtf(s[2] / (float)F + eps);
  const float c0 = coef[0], c1 = coef[1], c2 = coef[2], c3 = coef[3];
  for (int i = threadIdx.x * V; i < F; i += 256 * V) {
    float v[4], o[4];
    ldv<S, V>(zr + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float v2 = v[j] * v[j];
      o[j] = c0 * (v[j] * r1) + c1 * (v2 * r2) + c2 * (v2 * v[j] * r3) + c3;
    }
    stv<S, V>(out + (size_t)t * F + i, o);
  }
}

template <typename S, int V>
__global__ void __launch_bounds__(256) gated_residual_kernel(
    float* __restrict__ x, const S* __restrict__ a, float sa,
    const S* __restrict__ b, float sb, const S* __restrict__ g1, i64 ldg1,
    const float* __restrict__ b1, const S* __restrict__ m,
    const S* __restrict__ g2, i64 ldg2, const float* __restrict__ b2,
    int T, int W) {
  const i64 n = (i64)T * W;
  for (i64 i = ((i64)blockIdx.x * 256 + threadIdx.x) * V; i < n;
       i += (i64)gridDim.x * 256 * V) {
    const int t = (int)(i / W), c = (int)(i % W);
    float xv[4], av[4], bv[4] = {0.f, 0.f, 0.f, 0.f}, gv[4], bias[4], mv[4];
    ldv<float, V>(x + i, xv);
    ldv<S, V>(a + i, av);
    if (b) ldv<S, V>(b + i, bv);
    ldv<S, V>(g1 + (size_t)t * ldg1 + c, gv);
    ldv<float, V>(b1 + c, bias);
#pragma unroll
    for (int j = 0; j < V; ++j)
      xv[j] += (sa * av[j] + sb * bv[j]) / (1.0f + expf(-(gv[j] + bias[j])));
    if (m) {
      ldv<S, V>(m + i, mv);
      ldv<S, V>(g2 + (size_t)t * ldg2 + c, gv);
      ldv<float, V>(b2 + c, bias);
#pragma unroll
      for (int j = 0; j < V; ++j)
        xv[j] += mv[j] / (1.0f + expf(-(gv[j] + bias[j])));
    }
    stv<float, V>(x + i, xv);
  }
}

template <typename S>
__global__ void __launch_bounds__(256) softcap_kernel(
    float* __restrict__ out, const S* __restrict__ in, float cap, i64 n) {
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < n;
       i += (i64)gridDim.x * 256) {
    const float v = ldf<S>(in + i);
    out[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

// fp32 rows -> storage dtype (the projections' input when sublayers read the
// residual itself).
template <typename S>
__global__ void __launch_bounds__(256) cast_rows_kernel(
    S* __restrict__ out, const float* __restrict__ x, i64 n) {
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < n;
       i += (i64)gridDim.x * 256)
    stf<S>(out + i, x[i]);
}

// Norm on a sublayer's OUTPUT, then the residual add:
//   u = y (+ bias);  x += u / sqrt(mean(u^2) + eps) * w;  h = S(x)
// y is [T, W] in Y (storage dtype or fp32), x the fp32 residual, h an
// optional copy of the new residual row in the storage dtype.
template <typename S, typename Y, int V>
__global__ void __launch_bounds__(256) norm_residual_kernel(
    float* __restrict__ x, S* __restrict__ h, const Y* __restrict__ y,
    i64 ldy, const S* __restrict__ bias, const S* __restrict__ w, float eps,
    int W) {
  __shared__ float red[4];
  const int t = blockIdx.x;
  const Y* yr = y + (size_t)t * ldy;
  float ss[1] = {0.f};
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    float u[4], bv[4] = {0.f, 0.f, 0.f, 0.f};
    ldv<Y, V>(yr + i, u);
    if (bias) ldv<S, V>(bias + i, bv);
#pragma unroll
    for (int j = 0; j < V; ++j) { u[j] += bv[j]; ss[0] += u[j] * u[j]; }
  }
  block_sum<1>(ss, red);
  const float rs = 1.0f / sqrtf(ss[0] / (float)W + eps);
  float* xr = x + (size_t)t * W;
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    float u[4], bv[4] = {0.f, 0.f, 0.f, 0.f}, wv[4], xv[4];
    ldv<Y, V>(yr + i, u);
    if (bias) ldv<S, V>(bias + i, bv);
    ldv<S, V>(w + i, wv);
    ldv<float, V>(xr + i, xv);
#pragma unroll
    for (int j = 0; j < V; ++j) xv[j] += (u[j] + bv[j]) * rs * wv[j];
    stv<float, V>(xr + i, xv);
    if (h) stv<S, V>(h + (size_t)t * W + i, xv);
  }
}

// Gated linear unit over rows of [gate | up]:
//   out[r, i] = act(g[r, i] + bg[i]) * (u[r, i] + bu[i]) * rw[r]
// act: 0 SiLU, 1 ReLU, 2 tanh-GELU.  Biases and the per-row weight rw (fp32,
// e.g. a router weight per (token, expert) row) are optional.  Row r sits at
// (r / rg) * ld + (r % rg) * ld_in, so rg units laid side by side in one
// matrix row (experts of one token) are rows of their own.
template <typename S, int ACT, int V>
__global__ void __launch_bounds__(256) glu_kernel(
    S* __restrict__ out, i64 ldo, i64 ldo_in, const S* __restrict__ g,
    const S* __restrict__ u, i64 ldi, i64 ldi_in, int rg,
    const S* __restrict__ bg, const S* __restrict__ bu,
    const float* __restrict__ rw, i64 R, int F, float limit) {
  const int FV = F / V;
  const i64 n = R * FV;
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < n;
       i += (i64)gridDim.x * 256) {
    const i64 r = i / FV;
    const int c = (int)(i % FV) * V;
    const i64 ri = (r / rg) * ldi + (r % rg) * ldi_in;
    float a[4], b[4], ba[4] = {0.f, 0.f, 0.f, 0.f}, bb[4] = {0.f, 0.f, 0.f, 0.f};
    ldv<S, V>(g + ri + c, a);
    ldv<S, V>(u + ri + c, b);
    if (bg) ldv<S, V>(bg + c, ba);
    if (bu) ldv<S, V>(bu + c, bb);
    const float wr = rw ? rw[r] : 1.0f;
    float o[4];
#pragma unroll
    for (int j = 0; j < V; ++j) {
      float av = a[j] + ba[j];
      float uv = b[j] + bb[j];
      if (ACT == 0) av = av / (1.0f + expf(-av));
      else if (ACT == 1) av = fmaxf(av, 0.f);
      else if (ACT == 2)
        av = 0.5f * av * (1.0f + tanhf(0.7978845608028654f *
                                       (av + 0.044715f * av * av * av)));
      else {   // clamped unit: min(g, L) sigmoid(1.702 g) (clamp(u, -L, L) + 1)
        av = fminf(av, limit);
        av = av / (1.0f + expf(-1.702f * av));
        uv = fminf(fmaxf(uv, -limit), limit) + 1.0f;
      }
      o[j] = av * uv * wr;
    }
    stv<S, V>(out + (r / rg) * ldo + (r % rg) * ldo_in + c, o);
  }
}

// Router with score correction and group-limited top-k of one token by one
// wave.  zr [E] fp32 logits; s = sigmoid(z) or softmax(z) over all E; choice =
// s + corr.  With n_groups > 0 the experts form n_groups equal groups of
// neighbours, a group's score is the sum of its two largest choice scores (gtop
// 1: its largest choice score), and experts outside the best `keep` groups
// cannot be chosen.  The `top` largest choice scores win (ties: lower index);
// weights = s / (sum of chosen s + 1e-20) * scale (renorm 0: s * scale).
// Outputs idx [top] i32, wts [top] fp32 and, optionally, the dense form wd [E]
// fp32 (zero for experts not chosen).  sh: 3 * E + n_groups floats of LDS that
// belong to the wave.
struct RouteArgs {
  const float* corr;
  int E, top, n_groups, keep;
  float scale;
  int softmax, renorm, gtop;
};

__device__ __forceinline__ void route_row(const float* zr, float* sh, i32* idx,
                                          float* wts, float* wd,
                                          const RouteArgs& A) {
  const int E = A.E, lane = threadIdx.x & 63;
  float* sig = sh;             // [E]
  float* choice = sh + E;      // [E]
  i32* list = reinterpret_cast<i32*>(sh + 2 * E);   // [top]
  float* gsc = sh + 3 * E;     // [n_groups]
  float zmax = 0.f, zinv = 1.f;
  if (A.softmax) {
    zmax = -INFINITY;
    for (int e = lane; e < E; e += 64) zmax = fmaxf(zmax, zr[e]);
    zmax = wave_max_f32(zmax);
    float zs = 0.f;
    for (int e = lane; e < E; e += 64) zs += expf(zr[e] - zmax);
    zinv = 1.0f / wave_sum_f32(zs);
  }
  for (int e = lane; e < E; e += 64) {
    const float s = A.softmax ? expf(zr[e] - zmax) * zinv
                              : 1.0f / (1.0f + expf(-zr[e]));
    sig[e] = s;
    choice[e] = s + (A.corr ? A.corr[e] : 0.f);
  }
  __builtin_amdgcn_wave_barrier();
  if (A.n_groups > 0 && A.keep < A.n_groups) {
    const int size = E / A.n_groups;
    for (int g = lane; g < A.n_groups; g += 64) {
      float a = -INFINITY, b = -INFINITY;   // largest, second largest
      for (int m = 0; m < size; ++m) {
        const float c = choice[g * size + m];
        if (c > a) { b = a; a = c; }
        else if (c > b) b = c;
      }
      gsc[g] = size > 1 && A.gtop > 1 ? a + b : a;
    }
    __builtin_amdgcn_wave_barrier();
    for (int g = lane; g < A.n_groups; g += 64) {
      const float mine = gsc[g];
      int rank = 0;
      for (int o = 0; o < A.n_groups; ++o)
        rank += (gsc[o] > mine || (gsc[o] == mine && o < g)) ? 1 : 0;
      if (rank >= A.keep)
        for (int m = 0; m < size; ++m) choice[g * size + m] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
  }
  float total = 0.f;
  for (int r = 0; r < A.top; ++r) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float c = choice[e];
      if (c > bv) { bv = c; bi = e; }   // ascending e: first of equals stays
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    if (bi >= E) bi = r < E ? r : 0;    // fewer candidates than `top`
    total += sig[bi];
    __builtin_amdgcn_wave_barrier();
    if (lane == 0) {
      list[r] = bi;
      choice[bi] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
  }
  const float inv = A.renorm ? A.scale / (total + 1e-20f) : A.scale;
  for (int e = lane; e < E; e += 64) choice[e] = 0.f;     // now the dense form
  __builtin_amdgcn_wave_barrier();
  for (int r = lane; r < A.top; r += 64) {
    const int e = list[r];
    const float w = sig[e] * inv;
    idx[r] = e;
    wts[r] = w;
    choice[e] = w;
  }
  __builtin_amdgcn_wave_barrier();
  if (wd)
    for (int e = lane; e < E; e += 64) wd[e] = choice[e];
}

// One wave per token from ready logits z [T, E].
__global__ void __launch_bounds__(64) moe_route_kernel(
    i32* idx, float* wts, float* wd, const float* __restrict__ z, RouteArgs A) {
  extern __shared__ float sh[];
  const size_t t = blockIdx.x;
  route_row(z + t * A.E, sh, idx + t * A.top, wts + t * A.top,
            wd ? wd + t * A.E : nullptr, A);
}

// Router logits and routing of 16 tokens per workgroup of NW waves, bf16
// inputs: z = h R^T in fp32.  Wave w takes the 32-wide steps w, w + NW, .. of
// the inner dimension; h rows are A fragments, and the fp32 router weights
// enter as three bf16 terms (all 24 bits), so a product is exact and only the
// fp32 sums round.  The waves' sums meet in LDS, then wave w routes the tokens
// w, w + NW, ..  ET: 16-expert tiles.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

template <int ET, int NW>
__global__ void __launch_bounds__(NW * 64) moe_router_kernel(
    i32* idx, float* wts, float* wd, const u16* __restrict__ h, i64 ldh,
    const float* __restrict__ router, int T, int W, RouteArgs A) {
  constexpr int EP = ET * 16;
  extern __shared__ float sh[];            // [NW][16][EP], then the waves' rows
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int t0 = blockIdx.x * 16, E = A.E;
  const u16* hr = h + (size_t)min(t0 + (lane & 15), T - 1) * ldh;
  f32x4 acc[ET];
#pragma unroll
  for (int et = 0; et < ET; ++et) acc[et] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = wid * 32; k0 < W; k0 += NW * 32) {
    // loads without conditions, so that several steps' are in flight: past W
    // (a multiple of 8) the h fragment is zero, columns past E are never read
    const int k = k0 + (lane >> 4) * 8, kc = min(k, W - 8);
    union { s16x8 s; bf16x8 b; } a;
    a.s = *reinterpret_cast<const s16x8*>(hr + kc);
    if (k >= W) a.s = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int et = 0; et < ET; ++et) {
      const int n = min(et * 16 + (lane & 15), E - 1);
      const f32x4* rp = reinterpret_cast<const f32x4*>(router + (size_t)n * W + kc);
      const f32x4 r0 = rp[0], r1 = rp[1];
      float r[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) { r[j] = r0[j]; r[4 + j] = r1[j]; }
#pragma unroll
      for (int term = 0; term < 3; ++term) {
        bf16x8 b;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          b[j] = static_cast<__bf16>(r[j]);
          r[j] -= static_cast<float>(b[j]);
        }
        acc[et] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, b, acc[et], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int et = 0; et < ET; ++et)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      sh[(wid * 16 + (lane >> 4) * 4 + r) * EP + et * 16 + (lane & 15)] = acc[et][r];
  __syncthreads();
  float* mine = sh + NW * 16 * EP + wid * (4 * E + A.n_groups);
  for (int row = wid; row < 16; row += NW) {
    const size_t t = t0 + row;
    if (t >= (size_t)T) break;
    __builtin_amdgcn_wave_barrier();       // the previous token's row is read
    for (int e = lane; e < E; e += 64) {
      float z = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) z += sh[(w * 16 + row) * EP + e];
      mine[e] = z;
    }
    __builtin_amdgcn_wave_barrier();
    route_row(mine, mine + E, idx + t * A.top, wts + t * A.top,
              wd ? wd + t * E : nullptr, A);
  }
}

// y[t] = sum_r wts[t, r] * ys[pos[t*top + r]] (+ shared[t]) (+ (sum_i idw[t, i])
// hin[t]) in fp32, the sum taken in the order r = 0 .. top-1.  ys rows sit in
// expert-sorted order; pos is the inverse of that sort, negative for choices
// without a row.  idw [nid] at row stride ldi: the weights of experts whose
// output is their input hin.
template <typename S>
__global__ void __launch_bounds__(256) moe_combine_kernel(
    float* __restrict__ y, const S* __restrict__ ys,
    const i32* __restrict__ pos, const float* __restrict__ wts,
    const S* __restrict__ shared, const S* __restrict__ hin,
    const float* __restrict__ idw, i64 ldi, int nid, int top, int W) {
  const int t = blockIdx.x;
  float fid = 0.f;
  for (int i = 0; i < nid; ++i) fid += idw[(size_t)t * ldi + i];
  for (int i = threadIdx.x; i < W; i += 256) {
    float acc = shared ? ldf<S>(shared + (size_t)t * W + i) : 0.f;
    for (int r = 0; r < top; ++r) {
      const int p = pos[(size_t)t * top + r];
      if (p >= 0) acc += wts[(size_t)t * top + r] * ldf<S>(ys + (size_t)p * W + i);
    }
    if (fid != 0.f) acc += fid * ldf<S>(hin + (size_t)t * W + i);
    y[(size_t)t * W + i] = acc;
  }
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

AF_EXPORT int afm_embed(void* out, const void* table, const void* ids,
                        const void* add, float scale, int T, int W, int dt,
                        void* stream) {
  if (T == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  MIX_DISPATCH(dt,
      (embed_kernel<u16><<<T, 256, 0, s>>>((float*)out, (const u16*)table,
          (const i32*)ids, (const float*)add, scale, W)),
      (embed_kernel<float><<<T, 256, 0, s>>>((float*)out, (const float*)table,
          (const i32*)ids, (const float*)add, scale, W)));
  return af_last_err();
}

// prev [slots] i32; step: every chunk is one row.
AF_EXPORT int afm_embed_pairs(void* out, const void* table, const void* pairs,
                              const void* ids, void* prev, const void* row_seq,
                              const void* cu, const void* q_start,
                              const void* sslot, i64 mul_prev, i64 mul_cur,
                              i64 buckets, int T, int B, int W, int step,
                              int dt, void* stream) {
  if (T == 0) return 0;
  if (buckets < 1 || !prev) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = W % 4 == 0 && aligned16(out, table, pairs);
#define EP(ST, V, SP)                                                         \
  embed_pairs_kernel<ST, V, SP><<<T, 256, 0, s>>>((float*)out,                \
      (const ST*)table, (const ST*)pairs, (const i32*)ids, (i32*)prev,        \
      (const i32*)row_seq, (const i32*)cu, (const i32*)q_start,               \
      (const i32*)sslot, mul_prev, mul_cur, buckets, W)
#define EPV(ST)                                                               \
  do {                                                                        \
    if (vec) { if (step) EP(ST, 4, true); else EP(ST, 4, false); }            \
    else { if (step) EP(ST, 1, true); else EP(ST, 1, false); }                \
  } while (0)
  MIX_DISPATCH(dt, EPV(u16), EPV(float));
#undef EPV
#undef EP
  if (!step)
    last_token_kernel<<<(B + 255) / 256, 256, 0, s>>>(
        (i32*)prev, (const i32*)ids, (const i32*)cu, (const i32*)sslot, B);
  return af_last_err();
}

AF_EXPORT int afm_add_rows(void* x, const void* other, const void* vec, int T,
                           int W, void* stream) {
  if (T == 0) return 0;
  const i64 n = (i64)T * W;
  add_rows_kernel<<<grid_for(n), 256, 0, (hipStream_t)stream>>>(
      (float*)x, (const float*)other, (const float*)vec, n, W);
  return af_last_err();
}

AF_EXPORT int afm_dual_norm_shift(
    void* a, void* s_out, void* b, void* last, const void* x, const void* w1,
    const void* w2, const void* shift, const void* prev, const void* row_seq,
    const void* cu, const void* q_start, const void* sslot, float eps, int T,
    int W, int dt, void* stream) {
  if (T == 0) return 0;
  if (shift && !prev) return 9003;
  if ((b == nullptr) != (w2 == nullptr)) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = W % 4 == 0 && aligned16(a, s_out, b, last, x, w1) &&
                   aligned16(w2, shift, prev);
#define DNS(ST, V)                                                            \
  dual_norm_shift_kernel<ST, V><<<T, 256, 0, s>>>((ST*)a, (ST*)s_out, (ST*)b, \
      (float*)last, (const float*)x, (const ST*)w1, (const ST*)w2,            \
      (const ST*)shift, (float*)prev, (const i32*)row_seq,                    \
      (const i32*)cu, (const i32*)q_start, (const i32*)sslot, eps, W)
  if (vec) MIX_DISPATCH(dt, (DNS(u16, 4)), (DNS(float, 4)));
  else MIX_DISPATCH(dt, (DNS(u16, 1)), (DNS(float, 1)));
#undef DNS
  return af_last_err();
}

AF_EXPORT int afm_scatter_state(void* prev, const void* last,
                                const void* sslot, const void* cu, int B,
                                int W, void* stream) {
  if (B == 0) return 0;
  scatter_state_kernel<<<B, 256, 0, (hipStream_t)stream>>>(
      (float*)prev, (const float*)last, (const i32*)sslot, (const i32*)cu, W);
  return af_last_err();
}

AF_EXPORT int afm_norm_rows(void* out, const void* x, const void* w,
                            const void* rows, float eps, int R, int W,
                            int one_plus, int center, int dt, void* stream) {
  if (R == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  MIX_DISPATCH(dt,
      (norm_rows_kernel<u16><<<R, 256, 0, s>>>((u16*)out, (const float*)x,
          (const u16*)w, (const i32*)rows, eps, W, one_plus, center)),
      (norm_rows_kernel<float><<<R, 256, 0, s>>>((float*)out, (const float*)x,
          (const float*)w, (const i32*)rows, eps, W, one_plus, center)));
  return af_last_err();
}

AF_EXPORT int afm_headnorm_gate(void* out, const void* o, const void* g,
                                const void* w, float eps, int T, int H, int dv,
                                i64 ldg, int gate_act, int dt, void* stream) {
  if (T == 0) return 0;
  const int n_rh = T * H;
  const int grid = (n_rh + 3) / 4;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = dv % 4 == 0 && ldg % 4 == 0 && aligned16(out, o, g, w);
#define HG(ST, V, SG)                                                       \
  headnorm_gate_kernel<ST, V, SG><<<grid, 256, 0, s>>>((ST*)out,            \
      (const float*)o, (const ST*)g, (const ST*)w, eps, n_rh, H, dv, ldg)
  if (gate_act == 1) {
    if (vec) MIX_DISPATCH(dt, (HG(u16, 4, true)), (HG(float, 4, true)));
    else MIX_DISPATCH(dt, (HG(u16, 1, true)), (HG(float, 1, true)));
  } else {
    if (vec) MIX_DISPATCH(dt, (HG(u16, 4, false)), (HG(float, 4, false)));
    else MIX_DISPATCH(dt, (HG(u16, 1, false)), (HG(float, 1, false)));
  }
#undef HG
  return af_last_err();
}

AF_EXPORT int afm_polynorm(void* out, const void* z, const void* coef,
                           float eps, int T, int F, i64 ldz, int dt,
                           void* stream) {
  if (T == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = F % 4 == 0 && ldz % 4 == 0 && aligned16(out, z);
#define PN(ST, V)                                                     \
  polynorm_kernel<ST, V><<<T, 256, 0, s>>>((ST*)out, (const ST*)z,    \
      (const float*)coef, eps, F, ldz)
  if (vec) MIX_DISPATCH(dt, (PN(u16, 4)), (PN(float, 4)));
  else MIX_DISPATCH(dt, (PN(u16, 1)), (PN(float, 1)));
#undef PN
  return af_last_err();
}

AF_EXPORT int afm_gated_residual(
    void* x, const void* a, float sa, const void* b, float sb, const void* g1,
    i64 ldg1, const void* b1, const void* m, const void* g2, i64 ldg2,
    const void* b2, int T, int W, int dt, void* stream) {
  if (T == 0) return 0;
  if (m && (!g2 || !b2)) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = W % 4 == 0 && ldg1 % 4 == 0 && ldg2 % 4 == 0 &&
                   aligned16(x, a, b, g1, b1, m) && aligned16(g2, b2);
  const int grid = grid_for((i64)T * W / (vec ? 4 : 1));
#define GR(ST, V)                                                          \
  gated_residual_kernel<ST, V><<<grid, 256, 0, s>>>((float*)x,             \
      (const ST*)a, sa, (const ST*)b, sb, (const ST*)g1, ldg1,             \
      (const float*)b1, (const ST*)m, (const ST*)g2, ldg2, (const float*)b2, \
      T, W)
  if (vec) MIX_DISPATCH(dt, (GR(u16, 4)), (GR(float, 4)));
  else MIX_DISPATCH(dt, (GR(u16, 1)), (GR(float, 1)));
#undef GR
  return af_last_err();
}

AF_EXPORT int afm_softcap(void* out, const void* in, float cap, i64 n, int dt,
                          void* stream) {
  if (n == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  MIX_DISPATCH(dt,
      (softcap_kernel<u16><<<grid_for(n), 256, 0, s>>>((float*)out,
          (const u16*)in, cap, n)),
      (softcap_kernel<float><<<grid_for(n), 256, 0, s>>>((float*)out,
          (const float*)in, cap, n)));
  return af_last_err();
}

AF_EXPORT int afm_cast_rows(void* out, const void* x, i64 n, int dt,
                            void* stream) {
  if (n == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  MIX_DISPATCH(dt,
      (cast_rows_kernel<u16><<<grid_for(n), 256, 0, s>>>((u16*)out,
          (const float*)x, n)),
      (cast_rows_kernel<float><<<grid_for(n), 256, 0, s>>>((float*)out,
          (const float*)x, n)));
  return af_last_err();
}

// y_f32 != 0: y holds fp32 whatever the storage dtype.
AF_EXPORT int afm_norm_residual(void* x, void* h, const void* y, i64 ldy,
                                int y_f32, const void* bias, const void* w,
                                float eps, int T, int W, int dt,
                                void* stream) {
  if (T == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = W % 4 == 0 && ldy % 4 == 0 && aligned16(x, h, y, bias, w);
#define NR(ST, YT)                                                          \
  do {                                                                      \
    if (vec)                                                                \
      norm_residual_kernel<ST, YT, 4><<<T, 256, 0, s>>>((float*)x, (ST*)h,  \
          (const YT*)y, ldy, (const ST*)bias, (const ST*)w, eps, W);        \
    else                                                                    \
      norm_residual_kernel<ST, YT, 1><<<T, 256, 0, s>>>((float*)x, (ST*)h,  \
          (const YT*)y, ldy, (const ST*)bias, (const ST*)w, eps, W);        \
  } while (0)
  if (dt == 0) { if (y_f32) NR(u16, float); else NR(u16, u16); }
  else if (dt == 1) NR(float, float);
  else return 9002;
#undef NR
  return af_last_err();
}

// x [T, W] fp32 in place; y (or null) at row stride ldy, fp32 when y_f32; h
// (or null) [T, W] in the storage dtype.
AF_EXPORT int afm_sandwich_norm(void* x, void* h, const void* y, i64 ldy,
                                int y_f32, const void* w_post,
                                const void* w_pre, float mult, float eps,
                                int T, int W, int dt, void* stream) {
  if (T == 0) return 0;
  if ((y && !w_post) || (h && !w_pre)) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = W % 4 == 0 && ldy % 4 == 0 && aligned16(x, h, y, w_post, w_pre);
  const int cols = W / (vec ? 4 : 1);
  // few rows of many columns: one column group per thread
  const bool wide = T <= 512 && cols > 256;
#define SWK(ST, YT, V, NT, R)                                                \
  sandwich_norm_kernel<ST, YT, V, NT, R><<<T, NT, 0, s>>>((float*)x, (ST*)h, \
      (const YT*)y, ldy, (const ST*)w_post, (const ST*)w_pre, mult, eps, W)
#define SWR(ST, YT, V)                                                       \
  do {                                                                       \
    if (wide && cols <= SWN_IT * 1024) SWK(ST, YT, V, 1024, true);           \
    else if (!wide && cols <= SWN_IT * 256) SWK(ST, YT, V, 256, true);       \
    else SWK(ST, YT, V, 256, false);                                         \
  } while (0)
#define SW(ST, YT)                                                           \
  do { if (vec) SWR(ST, YT, 4); else SWR(ST, YT, 1); } while (0)
  if (dt == 0) { if (y_f32) SW(u16, float); else SW(u16, u16); }
  else if (dt == 1) SW(float, float);
  else return 9002;
#undef SW
#undef SWR
#undef SWK
  return af_last_err();
}

// x [T, W] fp32 in place; a at row stride lda, hin [T, W], ys rows of W in the
// storage dtype; h (or null) [T, W] in the storage dtype.
AF_EXPORT int afm_residual_norm(void* x, void* h, const void* a, i64 lda,
                                const void* parts, int np, const void* ys, const void* pos,
                                const void* wts, int top, const void* hin,
                                const void* idw, i64 ldi, int nid, float mult,
                                const void* vec, const void* w, float eps,
                                int T, int W, int dt, void* stream) {
  if (T == 0) return 0;
  if (h && !w) return 9003;
  if (np < 0 || (np > 0 && !parts)) return 9003;
  if (top < 0 || (top > 0 && (!ys || !pos || !wts))) return 9003;
  if (nid < 0 || (nid > 0 && (!hin || !idw))) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vv = W % 4 == 0 && lda % 4 == 0 &&
                  aligned16(x, h, a, ys, hin, vec, w) && aligned16(parts);
  const int cols = W / (vv ? 4 : 1);
  // few rows of many columns: one column group per thread
  const bool wide = T <= 512 && cols > 256;
#define RNK(ST, V, NT, R)                                                    \
  residual_norm_kernel<ST, V, NT, R><<<T, NT, 0, s>>>((float*)x, (ST*)h,     \
      (const ST*)a, lda, (const float*)parts, np, (const ST*)ys,             \
      (const i32*)pos, (const float*)wts, top, (const ST*)hin,               \
      (const float*)idw, ldi, nid, mult, (const float*)vec, (const ST*)w,    \
      eps, W)
#define RNR(ST, V)                                                           \
  do {                                                                       \
    if (wide && cols <= SWN_IT * 1024) RNK(ST, V, 1024, true);               \
    else if (!wide && cols <= SWN_IT * 256) RNK(ST, V, 256, true);           \
    else RNK(ST, V, 256, false);                                             \
  } while (0)
#define RN(ST)                                                               \
  do { if (vv) RNR(ST, 4); else RNR(ST, 1); } while (0)
  MIX_DISPATCH(dt, RN(u16), RN(float));
#undef RN
#undef RNR
#undef RNK
  return af_last_err();
}

// z, out [T, F] at row strides ldz, ldo; rw (or null) at row stride ldrw.
AF_EXPORT int afm_relu2(void* out, i64 ldo, const void* z, i64 ldz,
                        const void* rw, i64 ldrw, int lead, int unit, int T,
                        int F, int dt, void* stream) {
  if (T == 0 || F == 0) return 0;
  if (lead < 0 || unit < 1 ||
      (rw && F > lead && ((F - lead) % unit || ldrw < (F - lead) / unit)))
    return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = F % 4 == 0 && ldz % 4 == 0 && ldo % 4 == 0 &&
                   (!rw || (lead % 4 == 0 && unit % 4 == 0)) &&
                   (uintptr_t)out % (dt ? 16 : 8) == 0 &&
                   (uintptr_t)z % (dt ? 16 : 8) == 0;
  const i64 total = (i64)T * (vec ? F / 4 : F);
  const int grid = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
#define R2(S, V)                                                             \
  relu2_kernel<S, V><<<grid, 256, 0, s>>>((S*)out, ldo, (const S*)z, ldz,    \
      (const float*)rw, ldrw, lead, unit, T, F)
  if (dt == 0) { if (vec) R2(u16, 4); else R2(u16, 1); }
  else if (dt == 1) { if (vec) R2(float, 4); else R2(float, 1); }
  else return 9002;
#undef R2
  return af_last_err();
}

AF_EXPORT int afm_xielu(void* out, const void* z, i64 ldz, const void* coef,
                        int T, int F, int dt, void* stream) {
  if (T == 0 || F == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = F % 4 == 0 && ldz % 4 == 0 && aligned16(out, z);
  const i64 total = (i64)T * (vec ? F / 4 : F);
  const int grid = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
#define XI(S, V)                                                             \
  xielu_kernel<S, V><<<grid, 256, 0, s>>>((S*)out, (const S*)z, ldz,         \
                                          (const float*)coef, T, F)
  if (dt == 0) { if (vec) XI(u16, 4); else XI(u16, 1); }
  else if (dt == 1) { if (vec) XI(float, 4); else XI(float, 1); }
  else return 9002;
#undef XI
  return af_last_err();
}

AF_EXPORT int afm_glu(void* out, i64 ldo, i64 ldo_in, const void* g,
                      const void* u, i64 ldi, i64 ldi_in, int rg,
                      const void* bg, const void* bu, const void* rw, i64 R,
                      int F, int act, float limit, int dt, void* stream) {
  if (R == 0 || F == 0) return 0;
  if (act < 0 || act > 3 || rg < 1) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = F % 4 == 0 && ldo % 4 == 0 && ldo_in % 4 == 0 &&
                   ldi % 4 == 0 && ldi_in % 4 == 0 &&
                   aligned16(out, g, u, bg, bu);
  const int grid = grid_for(R * F / (vec ? 4 : 1));
#define GLU(ST, A)                                                         \
  do {                                                                     \
    if (vec)                                                               \
      glu_kernel<ST, A, 4><<<grid, 256, 0, s>>>((ST*)out, ldo, ldo_in,     \
          (const ST*)g, (const ST*)u, ldi, ldi_in, rg, (const ST*)bg,      \
          (const ST*)bu, (const float*)rw, R, F, limit);                          \
    else                                                                   \
      glu_kernel<ST, A, 1><<<grid, 256, 0, s>>>((ST*)out, ldo, ldo_in,     \
          (const ST*)g, (const ST*)u, ldi, ldi_in, rg, (const ST*)bg,      \
          (const ST*)bu, (const float*)rw, R, F, limit);                          \
  } while (0)
#define GLU_ACT(ST)                                   \
  do {                                                \
    if (act == 0) GLU(ST, 0);                         \
    else if (act == 1) GLU(ST, 1);                    \
    else if (act == 2) GLU(ST, 2);                    \
    else GLU(ST, 3);                                  \
  } while (0)
  MIX_DISPATCH(dt, GLU_ACT(u16), GLU_ACT(float));
#undef GLU_ACT
#undef GLU
  return af_last_err();
}

AF_EXPORT int afm_moe_route(void* idx, void* wts, void* wd, const void* z,
                            const void* corr, int T, int E, int top,
                            int n_groups, int keep, float scale, int softmax,
                            int renorm, int gtop, void* stream) {
  if (T == 0) return 0;
  if (gtop < 1 || gtop > 2) return 9003;
  if (E < 1 || top < 1 || top > E) return 9003;
  if (n_groups > 0 && (E % n_groups != 0 || keep < 1)) return 9003;
  const size_t sm = (size_t)(3 * E + (n_groups > 0 ? n_groups : 0)) *
                    sizeof(float);
  if (sm > 60000) return 9004;
  const RouteArgs A{(const float*)corr, E, top, n_groups, keep, scale, softmax,
                    renorm, gtop};
  moe_route_kernel<<<T, 64, sm, (hipStream_t)stream>>>(
      (i32*)idx, (float*)wts, (float*)wd, (const float*)z, A);
  return af_last_err();
}

// h [T, W] bf16 at row stride ldh, router [E, W] fp32; 9004: sizes the fused
// form does not take (the caller makes the logits itself).
AF_EXPORT int afm_moe_router(void* idx, void* wts, void* wd, const void* h,
                             i64 ldh, const void* router, const void* corr,
                             int T, int W, int E, int top, int n_groups,
                             int keep, float scale, int softmax, int renorm,
                             int gtop, void* stream) {
  if (T == 0) return 0;
  if (gtop < 1 || gtop > 2) return 9003;
  if (E < 1 || top < 1 || top > E) return 9003;
  if (n_groups > 0 && (E % n_groups != 0 || keep < 1)) return 9003;
  if (E > 128 || W % 8 || ldh % 8 || !aligned16(h, router)) return 9004;
  const RouteArgs A{(const float*)corr, E, top, n_groups, keep, scale, softmax,
                    renorm, gtop};
  const int grid = (T + 15) / 16;
#define MR(ET, NW)                                                           \
  moe_router_kernel<ET, NW><<<grid, NW * 64,                                 \
      (size_t)(NW * 16 * ET * 16 + NW * (4 * E + (n_groups > 0 ? n_groups : 0))) * \
          sizeof(float), (hipStream_t)stream>>>(                             \
      (i32*)idx, (float*)wts, (float*)wd, (const u16*)h, ldh,                \
      (const float*)router, T, W, A)
  if (E <= 16) MR(1, 16);
  else if (E <= 32) MR(2, 16);
  else if (E <= 64) MR(4, 8);
  else MR(8, 4);
#undef MR
  return af_last_err();
}

AF_EXPORT int afm_moe_combine(void* y, const void* ys, const void* pos,
                              const void* wts, const void* shared,
                              const void* hin, const void* idw, i64 ldi,
                              int nid, int T, int top, int W, int dt,
                              void* stream) {
  if (T == 0) return 0;
  if (top < 0 || nid < 0 || (nid > 0 && (!hin || !idw))) return 9003;
  if (top > 0 && (!ys || !pos || !wts)) return 9003;
  hipStream_t s = (hipStream_t)stream;
  MIX_DISPATCH(dt,
      (moe_combine_kernel<u16><<<T, 256, 0, s>>>((float*)y, (const u16*)ys,
          (const i32*)pos, (const float*)wts, (const u16*)shared,
          (const u16*)hin, (const float*)idw, ldi, nid, top, W)),
      (moe_combine_kernel<float><<<T, 256, 0, s>>>((float*)y, (const float*)ys,
          (const i32*)pos, (const float*)wts, (const float*)shared,
          (const float*)hin, (const float*)idw, ldi, nid, top, W)));
  return af_last_err();
}
