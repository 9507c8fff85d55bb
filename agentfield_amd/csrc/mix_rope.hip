// Row steps in front of rotary attention: the step's cos / sin table, and
// bias, per-head RMSNorm, partial rotary positions and the K/V page append
// in one pass over a row.
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
