// Row steps in front of rotary attention: the step's cos / sin table; bias,
// per-head RMSNorm, partial rotary positions and the K/V page append in one
// pass over a row; short causal convolutions over q, k and v, RMSNorm over the
// whole q and k rows, rotation and page append in one pass over a row.
//
// Storage dtype S is bf16 (raw u16) or fp32; statistics, angles and the
// rotation are fp32 (the table's angles double precision).
#include "mix_rows.h"

namespace {

// ------------------------------------------------ q/k prep for attention
// cos | sin of position * f_i per row, the product and the functions taken
// in double precision: tab [T, 2*half] fp32.  One table serves every layer
// of a step that rotates with the same frequencies.
__global__ void __launch_bounds__(256) rotary_table_kernel(
    float* __restrict__ tab, const i32* __restrict__ positions,
    const double* __restrict__ inv_freq, i64 n, int half) {
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < n;
       i += (i64)gridDim.x * 256) {
    const i64 t = i / half;
    const int j = (int)(i % half);
    const double a = (double)positions[t] * inv_freq[j];
    tab[t * 2 * half + j] = (float)cos(a);
    tab[t * 2 * half + half + j] = (float)sin(a);
  }
}

// One workgroup per row, one wave per head at a time.  Every q head and k
// head: + bias, RMSNorm over the head with a weight shared by heads, rotary
// positions on the first `rot` dims (dim i pairs with i + rot/2, or with
// `inter` dim 2i with 2i + 1) with the row's cos | sin from `tab`.  q goes to
// a contiguous [T, H*dk] buffer, k and v (+ bias) to their pages; the value
// heads GV may be fewer than the key heads G.  V2: two adjacent elements per
// lane and access (even sizes, 4- / 8-byte aligned rows).
template <typename S, bool V2>
__global__ void __launch_bounds__(256) qk_rope_cache_kernel(
    S* __restrict__ qo, const S* __restrict__ q, i64 ldq,
    const S* __restrict__ k, i64 ldk, const S* __restrict__ v, i64 ldv,
    const S* __restrict__ qb, const S* __restrict__ kb,
    const S* __restrict__ vb, const S* __restrict__ qw,
    const S* __restrict__ kw, const float* __restrict__ tab, int rot,
    S* __restrict__ kc, S* __restrict__ vc, const i64* __restrict__ slots,
    float eps, int H, int G, int GV, int dk, int dv, int page, int inter) {
  extern __shared__ float sm[];            // [4][dk]
  constexpr int E = V2 ? 2 : 1;
  const int half = rot / 2;
  const int t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const float* cs = tab + (size_t)t * rot;  // [half] cos, [half] sin
  const i64 sl = slots[t];
  const i64 pg = sl / page, off = sl % page;
  float* nb = sm + wave * dk;
  for (int u = wave; u < H + G; u += 4) {
    const bool isq = u < H;
    const int hh = isq ? u : u - H;
    const S* src = isq ? q + (size_t)t * ldq + (size_t)hh * dk
                       : k + (size_t)t * ldk + (size_t)hh * dk;
    const S* bias = isq ? qb : kb;
    const S* w = isq ? qw : kw;
    float ss = 0.f;
    for (int d = lane * E; d < dk; d += 64 * E) {
      float x0, x1, b0 = 0.f, b1 = 0.f;
      ld2<S, V2>(src + d, x0, x1);
      if (bias) ld2<S, V2>(bias + (size_t)hh * dk + d, b0, b1);
      x0 += b0;
      x1 += b1;
      nb[d] = x0;
      if (V2) nb[d + 1] = x1;
      ss += x0 * x0 + x1 * x1;
    }
    ss = wave_sum_f32(ss);
    const float r = w ? 1.0f / sqrtf(ss / (float)dk + eps) : 1.0f;
    for (int d = lane * E; d < dk; d += 64 * E) {
      float w0 = 1.f, w1 = 1.f;
      if (w) ld2<S, V2>(w + d, w0, w1);
      nb[d] = nb[d] * r * w0;              // each lane rewrites its own slots
      if (V2) nb[d + 1] = nb[d + 1] * r * w1;
    }
    __builtin_amdgcn_wave_barrier();       // partners come from other lanes
    S* dst = isq ? qo + ((size_t)t * H + hh) * dk
                 : kc + (((size_t)pg * G + hh) * page + off) * dk;
    if (isq || sl >= 0) {
      for (int d = lane * E; d < dk; d += 64 * E) {
        float o[2];
#pragma unroll
        for (int e = 0; e < E; ++e) {
          const int dd = d + e;
          float x = nb[dd];
          if (inter && dd < rot) {
            const float sn = cs[half + (dd >> 1)];
            x = x * cs[dd >> 1] + nb[dd ^ 1] * ((dd & 1) ? sn : -sn);
          } else if (dd < half) x = x * cs[dd] - nb[dd + half] * cs[half + dd];
          else if (dd < rot) x = x * cs[dd - half] + nb[dd - half] * cs[dd];
          o[e] = x;
        }
        st2<S, V2>(dst + d, o[0], V2 ? o[1] : 0.f);
      }
    }
    __builtin_amdgcn_wave_barrier();       // the buffer is reused
  }
  if (sl < 0) return;
  for (int i = threadIdx.x * E; i < GV * dv; i += 256 * E) {
    float x0, x1, b0 = 0.f, b1 = 0.f;
    ld2<S, V2>(v + (size_t)t * ldv + i, x0, x1);
    if (vb) ld2<S, V2>(vb + i, b0, b1);
    st2<S, V2>(vc + (((size_t)pg * GV + i / dv) * page + off) * dv + (i % dv),
               x0 + b0, x1 + b1);
  }
}

// The same for even head sizes up to 128 * NP with aligned rows: a lane owns
// NP element pairs of every head, so its norm weights, cos / sin factors and
// rotation partners are fixed for the row and sit in registers; the next
// head's values are loaded while the current head is reduced and rotated.
template <typename S, int NP>
__global__ void __launch_bounds__(256) qk_rope_cache_pairs_kernel(
    S* __restrict__ qo, const S* __restrict__ q, i64 ldq,
    const S* __restrict__ k, i64 ldk, const S* __restrict__ v, i64 ldv,
    const S* __restrict__ qb, const S* __restrict__ kb,
    const S* __restrict__ vb, const S* __restrict__ qw,
    const S* __restrict__ kw, const float* __restrict__ tab, int rot,
    S* __restrict__ kc, S* __restrict__ vc, const i64* __restrict__ slots,
    float eps, int H, int G, int GV, int dk, int dv, int page, int inter) {
  extern __shared__ float sm[];            // [4][dk]
  const int half = rot / 2;
  const int t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const float* cs = tab + (size_t)t * rot;
  const i64 sl = slots[t];
  const i64 pg = sl / page, off = sl % page;
  float* nb = sm + wave * dk;
  // per-lane constants of the row: o = n[d] * cc + n[pi] * sn
  float cc[NP][2], sn[NP][2], wq[NP][2], wk[NP][2];
  int pi[NP][2];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int d = lane * 2 + 128 * p;
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int dd = d + e;
      cc[p][e] = 1.f; sn[p][e] = 0.f; pi[p][e] = dd < dk ? dd : 0;
      if (inter && dd < rot) {
        const float s1 = cs[half + (dd >> 1)];
        cc[p][e] = cs[dd >> 1]; sn[p][e] = (dd & 1) ? s1 : -s1; pi[p][e] = dd ^ 1;
      } else if (dd < half) { cc[p][e] = cs[dd]; sn[p][e] = -cs[half + dd]; pi[p][e] = dd + half; }
      else if (dd < rot) { cc[p][e] = cs[dd - half]; sn[p][e] = cs[dd]; pi[p][e] = dd - half; }
    }
    wq[p][0] = wq[p][1] = wk[p][0] = wk[p][1] = 1.f;
    if (d < dk) {
      if (qw) ld2<S, true>(qw + d, wq[p][0], wq[p][1]);
      if (kw) ld2<S, true>(kw + d, wk[p][0], wk[p][1]);
    }
  }
  auto fetch = [&](int u, float (&x)[NP][2]) {
    const bool isq = u < H;
    const int hh = isq ? u : u - H;
    const S* src = isq ? q + (size_t)t * ldq + (size_t)hh * dk
                       : k + (size_t)t * ldk + (size_t)hh * dk;
    const S* bias = isq ? qb : kb;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = lane * 2 + 128 * p;
      x[p][0] = x[p][1] = 0.f;
      if (d < dk) {
        ld2<S, true>(src + d, x[p][0], x[p][1]);
        if (bias) {
          float b0, b1;
          ld2<S, true>(bias + (size_t)hh * dk + d, b0, b1);
          x[p][0] += b0;
          x[p][1] += b1;
        }
      }
    }
  };
  float cur[NP][2], nxt[NP][2];
  if (wave < H + G) fetch(wave, cur);
  for (int u = wave; u < H + G; u += 4) {
    if (u + 4 < H + G) fetch(u + 4, nxt);
    const bool isq = u < H;
    const int hh = isq ? u : u - H;
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) ss += cur[p][0] * cur[p][0] + cur[p][1] * cur[p][1];
    const float r = (isq ? qw : kw)
        ? 1.0f / sqrtf(wave_sum_f32(ss) / (float)dk + eps) : 1.0f;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = lane * 2 + 128 * p;
      if (d < dk) {
        nb[d] = cur[p][0] * r * (isq ? wq[p][0] : wk[p][0]);
        nb[d + 1] = cur[p][1] * r * (isq ? wq[p][1] : wk[p][1]);
      }
    }
    __builtin_amdgcn_wave_barrier();       // partners come from other lanes
    S* dst = isq ? qo + ((size_t)t * H + hh) * dk
                 : kc + (((size_t)pg * G + hh) * page + off) * dk;
    if (isq || sl >= 0) {
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const int d = lane * 2 + 128 * p;
        if (d < dk)
          st2<S, true>(dst + d, nb[d] * cc[p][0] + nb[pi[p][0]] * sn[p][0],
                       nb[d + 1] * cc[p][1] + nb[pi[p][1]] * sn[p][1]);
      }
    }
    __builtin_amdgcn_wave_barrier();       // the buffer is reused
#pragma unroll
    for (int p = 0; p < NP; ++p) { cur[p][0] = nxt[p][0]; cur[p][1] = nxt[p][1]; }
  }
  if (sl < 0) return;
  for (int i = threadIdx.x * 2; i < GV * dv; i += 512) {
    float x0, x1, b0 = 0.f, b1 = 0.f;
    ld2<S, true>(v + (size_t)t * ldv + i, x0, x1);
    if (vb) ld2<S, true>(vb + i, b0, b1);
    st2<S, true>(vc + (((size_t)pg * GV + i / dv) * page + off) * dv + (i % dv),
                 x0 + b0, x1 + b1);
  }
}

// ------------------------- convolution, whole-row norm, rotation, page append
// p [T, C] holds [q (H*dk) | k (G*dk) | v (G*dv)] per row at stride ldp.  Every
// channel is first convolved over time (taps tap-major in cw [taps, C]; inputs
// from before a chunk from the sequence's slot of `state` [slots, taps-1, C],
// oldest first; inputs before position 0 are zero), then the q row and the k
// row are RMS-normed as wholes (weights qw [H*dk], kw [G*dk]; null: no norm) and
// the first `rot` dims of every head are rotated (dim i with i + rot/2, the
// row's cos | sin in tab).  q goes to a contiguous [T, H*dk] buffer, k and v to
// their pages.  STEP: every chunk is one row, and the slot moves on to the last
// taps-1 inputs here.
struct ConvRopeArgs {
  const i32 *row_seq, *cu, *q_start, *sslot;
  const float* tab;
  const i64* slots;
  i64 ldp;
  float eps;
  int T, H, G, dk, dv, rot, page, taps, rows;
};

// One row per workgroup, any sizes.  LDS: the convolved q and k rows wait in
// LDS for the norm; otherwise they are evaluated again.
template <typename S, bool STEP, bool LDS>
__global__ void __launch_bounds__(256) conv_qk_rope_kernel(
    S* __restrict__ qo, const S* __restrict__ p, const S* __restrict__ cw,
    S* state, const S* __restrict__ qw, const S* __restrict__ kw,
    S* __restrict__ kc, S* __restrict__ vc, ConvRopeArgs A) {
  extern __shared__ float buf[];           // [nq + nk]
  __shared__ float red[8];
  const int nq = A.H * A.dk, nk = A.G * A.dk, nv = A.G * A.dv, C = nq + nk + nv;
  const int t = blockIdx.x, b = A.row_seq[t];
  const int k = t - A.cu[b], pos = A.q_start[b] + k;
  const int hist = A.taps - 1;
  S* st = state + (size_t)A.sslot[b] * hist * C;
  auto conv = [&](int c) {
    float acc = 0.f;
    for (int l = 0; l <= hist; ++l) {      // lag
      if (pos - l < 0) break;
      const float v = l <= k ? ldf<S>(p + (size_t)(t - l) * A.ldp + c)
                             : ldf<S>(st + (size_t)(hist - (l - k)) * C + c);
      acc += ldf<S>(cw + (size_t)(hist - l) * C + c) * v;
    }
    return acc;
  };
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x; c < nq + nk; c += 256) {
    const float v = conv(c);
    if (LDS) buf[c] = v;
    (c < nq ? sq : sk) += v * v;
  }
  sq = wave_sum_f32(sq);
  sk = wave_sum_f32(sk);
  if ((threadIdx.x & 63) == 0) {
    red[threadIdx.x >> 6] = sq;
    red[4 + (threadIdx.x >> 6)] = sk;
  }
  __syncthreads();
  const float rq = qw ? 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)nq + A.eps) : 1.f;
  const float rk = kw ? 1.0f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)nk + A.eps) : 1.f;
  auto normed = [&](int c) {
    const float v = LDS ? buf[c] : conv(c);
    if (c < nq) return qw ? v * rq * ldf<S>(qw + c) : v;
    return kw ? v * rk * ldf<S>(kw + c - nq) : v;
  };
  const float* cs = A.tab + (size_t)t * A.rot;  // [half] cos, [half] sin
  const int half = A.rot / 2;
  const i64 sl = A.slots[t];
  const i64 pg = sl / A.page, off = sl % A.page;
  for (int c = threadIdx.x; c < nq + nk; c += 256) {
    const int e = c < nq ? c : c - nq;
    const int d = e % A.dk;
    float x = normed(c);
    if (d < half) x = x * cs[d] - normed(c + half) * cs[half + d];
    else if (d < A.rot) x = x * cs[d - half] + normed(c - half) * cs[d];
    if (c < nq) stf<S>(qo + (size_t)t * nq + c, x);
    else if (sl >= 0)
      stf<S>(kc + (((size_t)pg * A.G + e / A.dk) * A.page + off) * A.dk + d, x);
  }
  if (sl >= 0)
    for (int e = threadIdx.x; e < nv; e += 256)
      stf<S>(vc + (((size_t)pg * A.G + e / A.dv) * A.page + off) * A.dv + e % A.dv,
             conv(nq + nk + e));
  if (STEP && hist > 0) {
    __syncthreads();                       // every thread has read the slot
    for (int c = threadIdx.x; c < C; c += 256)
      for (int j = 0; j < hist; ++j) {     // entry j: position pos - hist + 1 + j
        S v = S(0);
        if (pos - hist + 1 + j >= 0)
          v = j == hist - 1 ? p[(size_t)t * A.ldp + c] : st[(size_t)(j + 1) * C + c];
        st[(size_t)j * C + c] = v;
      }
  }
}

__device__ __forceinline__ short bf_bits(float f) {   // hardware rounding
  return __builtin_bit_cast(short, static_cast<__bf16>(f));
}

// A barrier for data that meets in LDS: global loads and stores stay in flight.
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// bf16 rows whose sizes are multiples of 4 (rot of 8): a thread owns NG groups
// of four channels over A.rows consecutive rows, so its taps, norm weights and
// the inputs behind the current row sit in registers; the next row is loaded
// while the current one is reduced and rotated.  The convolved rows times the
// norm weights meet their rotation partners in LDS, two rows in turn, which
// leaves one barrier a row.
template <int TAPS, int NG, int NT, bool STEP>
__global__ void __launch_bounds__(NT, NG <= 2 ? 4 : 2) conv_qk_rope_bf16_kernel(
    u16* __restrict__ qo, const u16* __restrict__ p, const u16* __restrict__ cw,
    u16* state, const u16* __restrict__ qw, const u16* __restrict__ kw,
    u16* __restrict__ kc, u16* __restrict__ vc, ConvRopeArgs A) {
  constexpr int HIST = TAPS - 1, NW = NT / 64;
  extern __shared__ __align__(16) float buf2[];      // [2][nq + nk]
  __shared__ float red[2][2][NW];
  const int nq = A.H * A.dk, nk = A.G * A.dk, nv = A.G * A.dv, nqk = nq + nk;
  const int C = nqk + nv, half = A.rot / 2;
  const int t0 = blockIdx.x * A.rows, t1 = min(A.T, t0 + A.rows);
  auto get = [](const u16* q) { return *reinterpret_cast<const s16x4*>(q); };
  const s16x4 zero = {0, 0, 0, 0}, one = {0x3f80, 0x3f80, 0x3f80, 0x3f80};

  s16x4 wt[NG][TAPS], hist[NG][HIST > 0 ? HIST : 1], nw[NG], cur[NG], nxt[NG];
  int dd[NG];            // dim inside the head
  int po[NG];            // k, v: head * page * dim + dim inside the page
#pragma unroll
  for (int g = 0; g < NG; ++g) {
    const int c = (g * NT + threadIdx.x) * 4;
    nw[g] = one;
    cur[g] = nxt[g] = zero;
    dd[g] = po[g] = 0;
    if (c >= C) continue;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) wt[g][j] = get(cw + (size_t)j * C + c);
    if (c < nq) {
      if (qw) nw[g] = get(qw + c);
      dd[g] = c % A.dk;
    } else if (c < nqk) {
      if (kw) nw[g] = get(kw + c - nq);
      dd[g] = (c - nq) % A.dk;
      po[g] = (c - nq) / A.dk * A.page * A.dk + dd[g];
    } else {
      const int e = c - nqk;
      po[g] = e / A.dv * A.page * A.dv + e % A.dv;
    }
    nxt[g] = get(p + (size_t)t0 * A.ldp + c);
  }
  for (int t = t0; t < t1; ++t) {
    const int b = A.row_seq[t];
    const int k = t - A.cu[b], pos = A.q_start[b] + k;
    u16* st = state + (size_t)A.sslot[b] * HIST * C;
    const i64 sl = A.slots[t];
    const uint32_t pg = (uint32_t)sl / (uint32_t)A.page, off = (uint32_t)sl % (uint32_t)A.page;
    float* row = buf2 + (size_t)((t - t0) & 1) * nqk;
    if (t == t0 || k == 0) {               // the inputs behind this row
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        const int c = (g * NT + threadIdx.x) * 4;
        if (c >= C) continue;
#pragma unroll
        for (int l = 1; l <= HIST; ++l)
          hist[g][l - 1] = pos - l < 0 ? zero
              : l <= k ? get(p + (size_t)(t - l) * A.ldp + c)
                       : get(st + (size_t)(HIST - (l - k)) * C + c);
      }
    }
    float acc[NG][4];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      const int c = (g * NT + threadIdx.x) * 4;
      cur[g] = nxt[g];
      if (c >= C) continue;
      if (t + 1 < t1) nxt[g] = get(p + (size_t)(t + 1) * A.ldp + c);
      float ss = 0.f;
      // the weights stay packed: unpacked for the whole loop they would take
      // the registers of two more waves
#pragma unroll
      for (int j = 0; j < TAPS; ++j) asm volatile("" : "+v"(wt[g][j]));
      asm volatile("" : "+v"(nw[g]));
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        float a = bf2f((u16)wt[g][HIST][j]) * bf2f((u16)cur[g][j]);
#pragma unroll
        for (int l = 1; l <= HIST; ++l)
          a += bf2f((u16)wt[g][HIST - l][j]) * bf2f((u16)hist[g][l - 1][j]);
        ss += a * a;
        acc[g][j] = a;
      }
      if (c < nqk) {
        (c < nq ? sq : sk) += ss;
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[g][j] *= bf2f((u16)nw[g][j]);
        *reinterpret_cast<f32x4*>(row + c) = f32x4{acc[g][0], acc[g][1], acc[g][2], acc[g][3]};
      } else if (sl >= 0) {
        const s16x4 o = {bf_bits(acc[g][0]), bf_bits(acc[g][1]), bf_bits(acc[g][2]), bf_bits(acc[g][3])};
        *reinterpret_cast<s16x4*>(vc + (size_t)pg * A.G * A.page * A.dv + po[g] + off * A.dv) = o;
      }
      if (STEP) {
#pragma unroll
        for (int j = 0; j < HIST; ++j)     // entry j keeps lag HIST - 1 - j
          *reinterpret_cast<s16x4*>(st + (size_t)j * C + c) =
              j == HIST - 1 ? cur[g] : hist[g][HIST - 2 - j];
      } else if (HIST > 0) {
#pragma unroll
        for (int l = HIST - 1; l > 0; --l) hist[g][l] = hist[g][l - 1];
        hist[g][0] = cur[g];
      }
    }
    sq = wave_sum_f32(sq);
    sk = wave_sum_f32(sk);
    float(*rd)[NW] = red[(t - t0) & 1];
    if ((threadIdx.x & 63) == 0) {
      rd[0][threadIdx.x >> 6] = sq;
      rd[1][threadIdx.x >> 6] = sk;
    }
    // the other buffer's readers are all past their row once this is passed
    lds_barrier();
    float rq = 1.f, rk = 1.f;
    {
      float a = 0.f, e = 0.f;
#pragma unroll
      for (int i = 0; i < NW; ++i) { a += rd[0][i]; e += rd[1][i]; }
      if (qw) rq = 1.0f / sqrtf(a / (float)nq + A.eps);
      if (kw) rk = 1.0f / sqrtf(e / (float)nk + A.eps);
    }
    const float* cs = A.tab + (size_t)t * A.rot;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      const int c = (g * NT + threadIdx.x) * 4;
      if (c >= nqk) continue;
      const int d = dd[g];
      if (d < A.rot) {
        const bool low = d < half;
        const f32x4 co = *reinterpret_cast<const f32x4*>(cs + (low ? d : d - half));
        const f32x4 si = *reinterpret_cast<const f32x4*>(cs + (low ? half + d : d));
        const f32x4 y = *reinterpret_cast<const f32x4*>(row + (low ? c + half : c - half));
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[g][j] = acc[g][j] * co[j] + (low ? -y[j] : y[j]) * si[j];
      }
      const float rs = c < nq ? rq : rk;
      const s16x4 o = {bf_bits(acc[g][0] * rs), bf_bits(acc[g][1] * rs),
                       bf_bits(acc[g][2] * rs), bf_bits(acc[g][3] * rs)};
      if (c < nq) *reinterpret_cast<s16x4*>(qo + (size_t)t * nq + c) = o;
      else if (sl >= 0)
        *reinterpret_cast<s16x4*>(kc + (size_t)pg * A.G * A.page * A.dk + po[g] + off * A.dk) = o;
    }
  }
}

}  // namespace

AF_EXPORT int afm_rotary_table(void* tab, const void* positions,
                               const void* inv_freq, int T, int half,
                               void* stream) {
  if (T == 0 || half == 0) return 0;
  const i64 n = (i64)T * half;
  rotary_table_kernel<<<grid_for(n), 256, 0, (hipStream_t)stream>>>(
      (float*)tab, (const i32*)positions, (const double*)inv_freq, n, half);
  return af_last_err();
}

AF_EXPORT int afm_qk_rope_cache(
    void* qo, const void* q, i64 ldq, const void* k, i64 ldk, const void* v,
    i64 ldv, const void* qb, const void* kb, const void* vb, const void* qw,
    const void* kw, const void* tab, int rot, void* kc, void* vc,
    const void* slots, float eps, int T, int H, int G, int GV, int dk, int dv,
    int page, int inter, int dt, void* stream) {
  if (T == 0) return 0;
  if (G < 1 || GV < 1) return 9003;
  if (rot < 0 || rot > dk || rot % 2 != 0 || (rot > 0 && !tab)) return 9003;
  const size_t smem = (size_t)(4 * dk) * sizeof(float);
  if (smem > 60000) return 9004;
  hipStream_t s = (hipStream_t)stream;
  const size_t al = dt == 0 ? 4 : 8;       // bytes of an element pair
  auto ok = [&](const void* p) { return (uintptr_t)p % al == 0; };
  const bool v2 = dk % 2 == 0 && dv % 2 == 0 && ldq % 2 == 0 && ldk % 2 == 0 &&
                  ldv % 2 == 0 && ok(qo) && ok(q) && ok(k) && ok(v) && ok(qb) &&
                  ok(kb) && ok(vb) && ok(qw) && ok(kw) && ok(kc) && ok(vc);
#define QRC(ST, V2)                                                          \
  qk_rope_cache_kernel<ST, V2><<<T, 256, smem, s>>>((ST*)qo, (const ST*)q,   \
      ldq, (const ST*)k, ldk, (const ST*)v, ldv, (const ST*)qb,              \
      (const ST*)kb, (const ST*)vb, (const ST*)qw, (const ST*)kw,            \
      (const float*)tab, rot, (ST*)kc, (ST*)vc, (const i64*)slots, eps, H,   \
      G, GV, dk, dv, page, inter)
#define QRP(ST, NPV)                                                         \
  qk_rope_cache_pairs_kernel<ST, NPV><<<T, 256, smem, s>>>((ST*)qo,          \
      (const ST*)q, ldq, (const ST*)k, ldk, (const ST*)v, ldv,               \
      (const ST*)qb, (const ST*)kb, (const ST*)vb, (const ST*)qw,            \
      (const ST*)kw, (const float*)tab, rot, (ST*)kc, (ST*)vc,               \
      (const i64*)slots, eps, H, G, GV, dk, dv, page, inter)
  if (v2 && dk <= 128) MIX_DISPATCH(dt, (QRP(u16, 1)), (QRP(float, 1)));
  else if (v2 && dk <= 256) MIX_DISPATCH(dt, (QRP(u16, 2)), (QRP(float, 2)));
  else if (v2) MIX_DISPATCH(dt, (QRC(u16, true)), (QRC(float, true)));
  else MIX_DISPATCH(dt, (QRC(u16, false)), (QRC(float, false)));
#undef QRP
#undef QRC
  return af_last_err();
}

// p [T, H*dk + G*dk + G*dv] at row stride ldp; state (or null when taps is 1)
// [slots, taps-1, H*dk + G*dk + G*dv]; step: every chunk is one row and the
// slots move on, otherwise the caller moves them (afm_conv_state).
AF_EXPORT int afm_conv_qk_rope_cache(
    void* qo, const void* p, i64 ldp, const void* cw, int taps, void* state,
    const void* row_seq, const void* cu, const void* q_start,
    const void* sslot, const void* qw, const void* kw, const void* tab,
    int rot, void* kc, void* vc, const void* slots, float eps, int T, int H,
    int G, int dk, int dv, int page, int step, int dt, void* stream) {
  if (T == 0) return 0;
  if (H < 1 || G < 1 || dk < 1 || dv < 1 || taps < 1) return 9003;
  if (taps > 1 && !state) return 9003;
  if (rot < 0 || rot > dk || rot % 2 != 0 || (rot > 0 && !tab)) return 9003;
  const int nq = H * dk, nk = G * dk, nv = G * dv, C = nq + nk + nv;
  if (ldp < C) return 9003;
  hipStream_t s = (hipStream_t)stream;
  ConvRopeArgs A{(const i32*)row_seq, (const i32*)cu, (const i32*)q_start,
                 (const i32*)sslot, (const float*)tab, (const i64*)slots, ldp,
                 eps, T, H, G, dk, dv, rot, page, taps, 1};
  auto al = [](const void* q, size_t n) { return (uintptr_t)q % n == 0; };
  const size_t sm2 = (size_t)2 * (nq + nk) * sizeof(float);
  const int groups = (C + 3) / 4;
  const int nt = step ? 1024 : 512, ng = (groups + nt - 1) / nt;
  const bool fast = dt == 0 && taps <= 4 && ng <= (step ? 2 : 4) &&
      dk % 4 == 0 && dv % 4 == 0 && ldp % 4 == 0 && rot % 8 == 0 &&
      sm2 <= 60000 && al(p, 8) && al(qo, 8) && al(cw, 8) && al(state, 8) &&
      al(qw, 8) && al(kw, 8) && al(kc, 8) && al(vc, 8) && al(tab, 16);
  if (fast) {
    if (!step) A.rows = T >= 8192 ? 8 : T >= 2048 ? 4 : T >= 512 ? 2 : 1;
    const int grid = (T + A.rows - 1) / A.rows;
#define CQF(TP, NG, NT, SP)                                                  \
  conv_qk_rope_bf16_kernel<TP, NG, NT, SP><<<grid, NT, sm2, s>>>((u16*)qo,   \
      (const u16*)p, (const u16*)cw, (u16*)state, (const u16*)qw,            \
      (const u16*)kw, (u16*)kc, (u16*)vc, A)
#define CQN(TP)                                                              \
  do {                                                                       \
    if (step) { if (ng <= 1) CQF(TP, 1, 1024, true); else CQF(TP, 2, 1024, true); } \
    else if (ng <= 1) CQF(TP, 1, 512, false);                                \
    else if (ng <= 2) CQF(TP, 2, 512, false);                                \
    else if (ng <= 3) CQF(TP, 3, 512, false);                                \
    else CQF(TP, 4, 512, false);                                             \
  } while (0)
    if (taps == 1) CQN(1);
    else if (taps == 2) CQN(2);
    else if (taps == 3) CQN(3);
    else CQN(4);
#undef CQN
#undef CQF
    return af_last_err();
  }
  const size_t sm = (size_t)(nq + nk) * sizeof(float);
  const bool lds = sm <= 60000;
#define CQ(ST, SP, L)                                                        \
  conv_qk_rope_kernel<ST, SP, L><<<T, 256, L ? sm : 0, s>>>((ST*)qo,         \
      (const ST*)p, (const ST*)cw, (ST*)state, (const ST*)qw, (const ST*)kw, \
      (ST*)kc, (ST*)vc, A)
#define CQL(ST)                                                              \
  do {                                                                       \
    if (step) { if (lds) CQ(ST, true, true); else CQ(ST, true, false); }     \
    else { if (lds) CQ(ST, false, true); else CQ(ST, false, false); }        \
  } while (0)
  MIX_DISPATCH(dt, CQL(u16), CQL(float));
#undef CQL
#undef CQ
  return af_last_err();
}
