// Real-gated linear recurrent unit over packed row chunks, one fp32 state
// value per channel and sequence slot:
//
//   r = sigmoid(Wr_b u_b + br),  i = sigmoid(Wi_b u_b + bi)   per block b of channels
//   log a = rate * r             (rate = -c softplus(lambda), given per channel)
//   S <- a S + sqrt(1 - a^2) i u;   out = S * gelu_tanh(y + by)
//
//   rglru_gates    u [T, C] -> (a, sqrt(1 - a^2) i u) as fp32 pairs [T, C, 2];
//                  bf16 storage multiplies on the matrix cores, the gate
//                  logits stay fp32
//   rglru_scan     the recurrence along every chunk and the output gate
//   rglru_step     decode steps (one row per sequence): short convolution
//                  from the slot, gates, recurrence, output gate, both slot
//                  updates
//
// Storage dtype S is bf16 (raw u16) or fp32; gates, decays, the state and
// the products that enter it are fp32.
#include "mix_rows.h"

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

__device__ __forceinline__ bf16x8 as_bf16x8(s16x8 v) {
  union { s16x8 s; bf16x8 b; } u;
  u.s = v;
  return u.b;
}

// 8 consecutive bf16 from element e0 of a row of n elements, zero past n;
// VEC: e0 and n are multiples of 8 and the row is 16-byte aligned.
template <bool VEC>
__device__ __forceinline__ s16x8 load8(const u16* row, int e0, int n) {
  s16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
  if (VEC) {
    if (e0 < n) v = *reinterpret_cast<const s16x8*>(row + e0);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (e0 + j < n) v[j] = (short)row[e0 + j];
  }
  return v;
}

// Decay and input gain of one element.  1 - a^2 = -expm1(2 log a): fp32
// storage takes the library forms; bf16 storage the hardware exponential,
// reciprocal and root (one unit in the last fp32 place), with the series of
// expm1 near zero where the subtraction would cancel.
template <typename S>
__device__ __forceinline__ void decay_gain(float zr, float zi, float rate,
                                           float u, float& a, float& g) {
  if constexpr (sizeof(S) == 2) {
    const float la = rate * __builtin_amdgcn_rcpf(1.0f + __expf(-zr));
    const float gi = __builtin_amdgcn_rcpf(1.0f + __expf(-zi));
    const float z = 2.0f * la;
    a = __expf(la);
    const float q = z > -0.0625f
        ? -z * (1.0f + z * (0.5f + z * (0.16666667f + z * 0.041666668f)))
        : 1.0f - __expf(z);
    g = __builtin_amdgcn_sqrtf(q) * gi * u;
  } else {
    const float la = rate / (1.0f + expf(-zr));
    a = expf(la);
    g = sqrtf(-expm1f(2.0f * la)) * u / (1.0f + expf(-zi));
  }
}

// ------------------------------------------------------------------- gates
// Workgroup = 16*RT rows x one block of n channels.  The rows' channels sit
// in LDS as A rows; wave w takes the 16-column tiles w, w + 4, ... of both
// gate matrices (a B fragment is 16 contiguous bytes of a weight row, read
// from global memory), so that r and i of an element meet in one lane.
template <int RT, bool VEC>
__global__ void __launch_bounds__(256) rglru_gates_mfma_kernel(
    f32x2* __restrict__ ag, const u16* __restrict__ u, const u16* __restrict__ wr,
    const float* __restrict__ br, const u16* __restrict__ wi,
    const float* __restrict__ bi, const float* __restrict__ rate, int T, int C,
    int n) {
  extern __shared__ __align__(16) u16 us[];   // [16*RT][ks]
  const int kc = (n + 31) / 32, ks = kc * 32 + 8;
  const int t0 = blockIdx.x * 16 * RT, c0 = blockIdx.y * n;
  for (int i = threadIdx.x; i < 16 * RT * kc * 4; i += 256) {
    const int row = i / (kc * 4), e0 = (i % (kc * 4)) * 8;
    s16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
    if (t0 + row < T) v = load8<VEC>(u + (size_t)(t0 + row) * C + c0, e0, n);
    *reinterpret_cast<s16x8*>(us + row * ks + e0) = v;
  }
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int ln = lane & 15, lq = lane >> 4;
  const u16* wrb = wr + (size_t)blockIdx.y * n * n;
  const u16* wib = wi + (size_t)blockIdx.y * n * n;
  for (int nt = wave; nt * 16 < n; nt += 4) {
    const int col = nt * 16 + ln, cw = min(col, n - 1);
    f32x4 ar[RT], ai[RT];
#pragma unroll
    for (int m = 0; m < RT; ++m)
      ar[m] = ai[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < kc; ++k) {
      const s16x8 fr = load8<VEC>(wrb + (size_t)cw * n, k * 32 + lq * 8, n);
      const s16x8 fi = load8<VEC>(wib + (size_t)cw * n, k * 32 + lq * 8, n);
#pragma unroll
      for (int m = 0; m < RT; ++m) {
        const s16x8 fa = *reinterpret_cast<const s16x8*>(
            us + (m * 16 + ln) * ks + k * 32 + lq * 8);
        ar[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            as_bf16x8(fa), as_bf16x8(fr), ar[m], 0, 0, 0);
        ai[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            as_bf16x8(fa), as_bf16x8(fi), ai[m], 0, 0, 0);
      }
    }
    if (col >= n) continue;
    const float b0 = br[c0 + col], b1 = bi[c0 + col], rt = rate[c0 + col];
    const bool full = t0 + 16 * RT <= T;
    f32x2* dst = ag + (size_t)(t0 + lq * 4) * C + c0 + col;
#pragma unroll
    for (int m = 0; m < RT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = m * 16 + lq * 4 + r;
        if (!full && t0 + row >= T) continue;
        float a, g;
        decay_gain<u16>(ar[m][r] + b0, ai[m][r] + b1, rt,
                        bf2f(us[row * ks + col]), a, g);
        dst[(size_t)(m * 16 + r) * C] = f32x2{a, g};
      }
  }
}

// Plain form for fp32 storage and blocks past the tile kernel's LDS: 8 rows x
// one block per workgroup, a thread per output channel, the rows' channels
// staged GK at a time.
constexpr int GR = 8, GK = 512;

template <typename S>
__global__ void __launch_bounds__(256) rglru_gates_kernel(
    f32x2* __restrict__ ag, const S* __restrict__ u, const S* __restrict__ wr,
    const float* __restrict__ br, const S* __restrict__ wi,
    const float* __restrict__ bi, const float* __restrict__ rate, int T, int C,
    int n) {
  __shared__ float us[GR][GK];
  const int t0 = blockIdx.x * GR, c0 = blockIdx.y * n;
  const S* wrb = wr + (size_t)blockIdx.y * n * n;
  const S* wib = wi + (size_t)blockIdx.y * n * n;
  for (int cb = 0; cb < n; cb += 256) {
    const int col = cb + threadIdx.x;
    float zr[GR], zi[GR];
#pragma unroll
    for (int m = 0; m < GR; ++m) zr[m] = zi[m] = 0.f;
    for (int k0 = 0; k0 < n; k0 += GK) {
      const int kn = min(GK, n - k0);
      __syncthreads();
      for (int i = threadIdx.x; i < GR * kn; i += 256) {
        const int m = i / kn, k = i % kn;
        us[m][k] = t0 + m < T ? ldf<S>(u + (size_t)(t0 + m) * C + c0 + k0 + k) : 0.f;
      }
      __syncthreads();
      if (col < n) {
        const S* pr = wrb + (size_t)col * n + k0;
        const S* pi = wib + (size_t)col * n + k0;
        for (int k = 0; k < kn; ++k) {
          const float w0 = ldf<S>(pr + k), w1 = ldf<S>(pi + k);
#pragma unroll
          for (int m = 0; m < GR; ++m) {
            zr[m] += w0 * us[m][k];
            zi[m] += w1 * us[m][k];
          }
        }
      }
    }
    if (col < n) {
#pragma unroll
      for (int m = 0; m < GR; ++m) {
        if (t0 + m >= T) continue;
        const size_t o = (size_t)(t0 + m) * C + c0 + col;
        float a, g;
        decay_gain<S>(zr[m] + br[c0 + col], zi[m] + bi[c0 + col],
                      rate[c0 + col], ldf<S>(u + o), a, g);
        ag[o] = f32x2{a, g};
      }
    }
  }
}

// -------------------------------------------------------------------- scan
// Workgroup = (64 channels, sequence), lane = channel, NW waves.  Tokens
// advance NW*SEG at a time: wave w loads the SEG tokens of its segment into
// registers, composes them (the decays' product and the state they would
// leave behind from zero), and after one barrier every wave walks the
// composed segments in front of its own to its incoming state and replays
// its tokens from it; the next pass's decays and gains are in flight
// meanwhile.  The order of all sums is fixed.
constexpr int SEG = 16;

template <typename S, int NW>
__global__ void __launch_bounds__(64 * NW) rglru_scan_kernel(
    S* __restrict__ out, float* __restrict__ state,
    const f32x2* __restrict__ ag, const S* __restrict__ y, i64 ldy, const S* __restrict__ by,
    const i32* __restrict__ cu, const i32* __restrict__ q_start,
    const i32* __restrict__ sslot, int C) {
  __shared__ float sa[2][NW][64], sg[2][NW][64];
  const int b = blockIdx.y;
  const int r0 = cu[b], L = cu[b + 1] - r0;
  if (L == 0) return;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int c = blockIdx.x * 64 + lane;
  const bool ok = c < C;
  float* sp = state + (size_t)sslot[b] * C + c;
  float st = (ok && q_start[b] > 0) ? *sp : 0.f;
  const float bias = (ok && by) ? ldf<S>(by + c) : 0.f;
  int buf = 0;
  f32x2 nx[SEG];
  // whole segments load without a condition per token (lanes past C read the
  // last channel and write nothing)
  const int cl = min(c, C - 1);
  auto fetch = [&](int s0) {
    const f32x2* p = ag + (size_t)(r0 + s0) * C + cl;
    if (s0 + SEG <= L) {
#pragma unroll
      for (int i = 0; i < SEG; ++i) nx[i] = p[(size_t)i * C];
    } else {
#pragma unroll
      for (int i = 0; i < SEG; ++i) {
        nx[i] = f32x2{1.f, 0.f};
        if (s0 + i < L) nx[i] = p[(size_t)i * C];
      }
    }
  };
  fetch(wave * SEG);
  for (int tb = 0; tb < L; tb += NW * SEG, buf ^= 1) {
    const int s0 = tb + wave * SEG;              // this wave's tokens
    const int nt = min(SEG, L - s0);             // may be <= 0
    float av[SEG], gv[SEG];
    S yv[SEG];
#pragma unroll
    for (int i = 0; i < SEG; ++i) {
      av[i] = nx[i][0];
      gv[i] = nx[i][1];
    }
    const S* yp = y + (size_t)(r0 + s0) * ldy + cl;
    if (nt == SEG) {
#pragma unroll
      for (int i = 0; i < SEG; ++i) yv[i] = yp[i * ldy];
    } else {
#pragma unroll
      for (int i = 0; i < SEG; ++i) {
        yv[i] = S(0);
        if (i < nt) yv[i] = yp[i * ldy];
      }
    }
    if (tb + NW * SEG < L) fetch(s0 + NW * SEG);
    if constexpr (NW > 1) {
      float pa = 1.f, pg = 0.f;
#pragma unroll
      for (int i = 0; i < SEG; ++i) {
        pg = av[i] * pg + gv[i];
        pa *= av[i];
      }
      sa[buf][wave][lane] = pa;
      sg[buf][wave][lane] = pg;
      __syncthreads();    // double buffer: one barrier per pass is enough
    }
    float cur = st;
    if constexpr (NW > 1) {
      float mine = st;
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        if (w == wave) mine = st;
        st = sa[buf][w][lane] * st + sg[buf][w][lane];
      }
      cur = mine;
    }
    S* op = out + (size_t)(r0 + s0) * C + cl;
    if (nt == SEG) {
#pragma unroll
      for (int i = 0; i < SEG; ++i) {
        cur = av[i] * cur + gv[i];
        const float o = cur * gelu_tanh<S>(ldf<S>(&yv[i]) + bias);
        if (ok) stf<S>(op + (size_t)i * C, o);
      }
    } else {
#pragma unroll
      for (int i = 0; i < SEG; ++i) {
        if (i < nt) {
          cur = av[i] * cur + gv[i];
          if (ok)
            stf<S>(op + (size_t)i * C,
                   cur * gelu_tanh<S>(ldf<S>(&yv[i]) + bias));
        }
      }
    }
    // the state that goes on is the replayed one where this wave has it
    if constexpr (NW == 1) st = cur;
    else if (ok && nt > 0 && s0 + nt == L) *sp = cur;
  }
  if (NW == 1 && ok) *sp = st;
}

// -------------------------------------------------------------------- step
// Decode: row t is sequence t.  Workgroup = 16 rows x one block of n
// channels; it owns their convolution inputs and states, so both slots are
// moved in place.  The convolved rows meet in LDS, the gates run as in
// rglru_gates_mfma_kernel with NW waves.
// VEC: rows of 8 aligned elements for the weights, V = 4 channels per access
// in the convolution.
template <int NW, bool VEC>
__global__ void __launch_bounds__(64 * NW) rglru_step_kernel(
    u16* __restrict__ out, float* __restrict__ state, u16* __restrict__ hist,
    const u16* __restrict__ x, i64 ldx, const u16* __restrict__ bx,
    const u16* __restrict__ cw, const u16* __restrict__ cb,
    const u16* __restrict__ y, i64 ldy, const u16* __restrict__ by,
    const u16* __restrict__ wr, const float* __restrict__ br,
    const u16* __restrict__ wi, const float* __restrict__ bi,
    const float* __restrict__ rate, const i32* __restrict__ q_start,
    const i32* __restrict__ sslot, int B, int C, int n, int taps) {
  constexpr int V = VEC ? 4 : 1;
  extern __shared__ __align__(16) u16 us[];   // [16][ks]
  const int kc = (n + 31) / 32, ks = kc * 32 + 8;
  const int t0 = blockIdx.x * 16, c0 = blockIdx.y * n;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int ln = lane & 15, lq = lane >> 4;
  const u16* wrb = wr + (size_t)blockIdx.y * n * n;
  const u16* wib = wi + (size_t)blockIdx.y * n * n;
  // the first column tile's weights are in flight during the convolution
  constexpr int KP = 4;
  s16x8 pr[KP], pi[KP];
  if (wave * 16 < n) {
    const int cc = min(wave * 16 + ln, n - 1);
#pragma unroll
    for (int k = 0; k < KP; ++k) {          // zero past the row's end
      pr[k] = load8<VEC>(wrb + (size_t)cc * n, k * 32 + lq * 8, n);
      pi[k] = load8<VEC>(wib + (size_t)cc * n, k * 32 + lq * 8, n);
    }
  }
  for (int i = threadIdx.x * V; i < 16 * kc * 32; i += 64 * NW * V) {
    const int row = i / (kc * 32), k = i % (kc * 32);
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    const int t = t0 + row;
    if (t < B && k < n) {
      const int c = c0 + k;
      const int pos = q_start[t];
      u16* hp = hist + (size_t)sslot[t] * (taps - 1) * C + c;
      float xn[4], b[4] = {0.f, 0.f, 0.f, 0.f}, w[4], o[4];
      ldv<u16, V>(x + (size_t)t * ldx + c, xn);
      if (bx) ldv<u16, V>(bx + c, b);
      if (cb) ldv<u16, V>(cb + c, v);
      ldv<u16, V>(cw + (size_t)(taps - 1) * C + c, w);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] += w[j] * (xn[j] + b[j]);
      // lag l sits in history place taps-1-l and moves one place down
      float nw[4] = {xn[0], xn[1], xn[2], xn[3]};
      for (int l = 1; l < taps; ++l) {
        ldv<u16, V>(hp + (size_t)(taps - 1 - l) * C, o);
        stv<u16, V>(hp + (size_t)(taps - 1 - l) * C, nw);
        if (pos - l >= 0) {
          ldv<u16, V>(cw + (size_t)(taps - 1 - l) * C + c, w);
#pragma unroll
          for (int j = 0; j < V; ++j) v[j] += w[j] * (o[j] + b[j]);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) nw[j] = o[j];
      }
    }
    stv<u16, V>(us + row * ks + k, v);
  }
  __syncthreads();
  for (int nt = wave; nt * 16 < n; nt += NW) {
    const int col = nt * 16 + ln, cc = min(col, n - 1);
    f32x4 ar = f32x4{0.f, 0.f, 0.f, 0.f}, ai = ar;
    if (nt == wave) {
#pragma unroll
      for (int k = 0; k < KP; ++k) {
        if (k >= kc) break;
        const s16x8 fa = *reinterpret_cast<const s16x8*>(us + ln * ks + k * 32 + lq * 8);
        ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(fa), as_bf16x8(pr[k]), ar, 0, 0, 0);
        ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(fa), as_bf16x8(pi[k]), ai, 0, 0, 0);
      }
    }
    for (int k = nt == wave ? KP : 0; k < kc; ++k) {
      const s16x8 fr = load8<VEC>(wrb + (size_t)cc * n, k * 32 + lq * 8, n);
      const s16x8 fi = load8<VEC>(wib + (size_t)cc * n, k * 32 + lq * 8, n);
      const s16x8 fa = *reinterpret_cast<const s16x8*>(us + ln * ks + k * 32 + lq * 8);
      ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(fa), as_bf16x8(fr), ar, 0, 0, 0);
      ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(fa), as_bf16x8(fi), ai, 0, 0, 0);
    }
    if (col >= n) continue;
    const int c = c0 + col;
    const float b0 = br[c], b1 = bi[c], rt = rate[c];
    const float yb = by ? bf2f(by[c]) : 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = lq * 4 + r, t = t0 + row;
      if (t >= B) continue;
      float a, g;
      decay_gain<u16>(ar[r] + b0, ai[r] + b1, rt, bf2f(us[row * ks + col]), a, g);
      float* sp = state + (size_t)sslot[t] * C + c;
      const float s = a * (q_start[t] > 0 ? *sp : 0.f) + g;
      *sp = s;
      out[(size_t)t * C + c] =
          f2bf(s * gelu_tanh<u16>(bf2f(y[(size_t)t * ldy + c]) + yb));
    }
  }
}

template <typename S>
int launch_gates_plain(void* ag, const void* u, const void* wr,
                       const void* br, const void* wi, const void* bi,
                       const void* rate, int T, int C, int blocks,
                       hipStream_t s) {
  rglru_gates_kernel<S><<<dim3((T + GR - 1) / GR, blocks), 256, 0, s>>>(
      (f32x2*)ag, (const S*)u, (const S*)wr, (const float*)br,
      (const S*)wi, (const float*)bi, (const float*)rate, T, C, C / blocks);
  return af_last_err();
}

}  // namespace

// u [T, C] contiguous; wr, wi [blocks, n, n] ([out, in], n = C / blocks) in
// the storage dtype; br, bi, rate [C] fp32; ag [T, C, 2] fp32.
AF_EXPORT int afm_rglru_gates(void* ag, const void* u, const void* wr,
                              const void* br, const void* wi, const void* bi,
                              const void* rate, int T, int C, int blocks,
                              int dt, void* stream) {
  if (T == 0) return 0;
  if (blocks < 1 || C % blocks) return 9003;
  hipStream_t s = (hipStream_t)stream;
  const int n = C / blocks;
  if (dt == 1)
    return launch_gates_plain<float>(ag, u, wr, br, wi, bi, rate, T, C, blocks, s);
  if (dt != 0) return 9002;
  const int ks = (n + 31) / 32 * 32 + 8;
  const int rt = (T > 512 && (size_t)64 * ks * sizeof(u16) <= 65536) ? 4 : 1;
  const size_t sm = (size_t)16 * rt * ks * sizeof(u16);
  if (sm > 65536)
    return launch_gates_plain<u16>(ag, u, wr, br, wi, bi, rate, T, C, blocks, s);
  const bool vec = n % 8 == 0 && aligned16(u, wr, wi);
  const dim3 grid((T + 16 * rt - 1) / (16 * rt), blocks);
#define RG(RT, V)                                                             \
  rglru_gates_mfma_kernel<RT, V><<<grid, 256, sm, s>>>((f32x2*)ag,            \
      (const u16*)u, (const u16*)wr, (const float*)br, (const u16*)wi,        \
      (const float*)bi, (const float*)rate, T, C, n)
  if (rt == 4) { if (vec) RG(4, true); else RG(4, false); }
  else { if (vec) RG(1, true); else RG(1, false); }
#undef RG
  return af_last_err();
}

// out [T, C] in the storage dtype; y [T, C] at row stride ldy, by [C] (or
// null); state [slots, C] fp32; max_len: rows of the longest chunk.
AF_EXPORT int afm_rglru_scan(void* out, void* state, const void* ag,
                             const void* y, i64 ldy,
                             const void* by, const void* cu,
                             const void* q_start, const void* sslot, int B,
                             int C, int max_len, int dt, void* stream) {
  if (B == 0 || C == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((C + 63) / 64, B);
#define SC(ST, NW)                                                            \
  rglru_scan_kernel<ST, NW><<<grid, 64 * NW, 0, s>>>((ST*)out, (float*)state, \
      (const f32x2*)ag, (const ST*)y, ldy, (const ST*)by,                     \
      (const i32*)cu, (const i32*)q_start, (const i32*)sslot, C)
#define SCN(ST)                                                               \
  do {                                                                        \
    if (max_len <= SEG) SC(ST, 1);                                            \
    else if (max_len <= 4 * SEG) SC(ST, 4);                                   \
    else SC(ST, 16);                                                          \
  } while (0)
  MIX_DISPATCH(dt, SCN(u16), SCN(float));
#undef SCN
#undef SC
  return af_last_err();
}

// One row per sequence, bf16: x, y [B, C] at row strides ldx, ldy; hist
// [slots, taps-1, C]; cw tap-major [taps, C]; state [slots, C] fp32.  9004:
// the block does not fit the kernel's LDS tile (callers take the separate
// steps).
AF_EXPORT int afm_rglru_step(void* out, void* state, void* hist,
                             const void* x, i64 ldx, const void* bx,
                             const void* cw, const void* cb, const void* y,
                             i64 ldy, const void* by, const void* wr,
                             const void* br, const void* wi, const void* bi,
                             const void* rate, const void* q_start,
                             const void* sslot, int B, int C, int blocks,
                             int taps, void* stream) {
  if (B == 0) return 0;
  if (blocks < 1 || C % blocks || taps < 1 || (taps > 1 && !hist)) return 9003;
  const int n = C / blocks;
  const int ks = (n + 31) / 32 * 32 + 8;
  const size_t sm = (size_t)16 * ks * sizeof(u16);
  if (sm > 65536) return 9004;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = n % 8 == 0 && ldx % 4 == 0 &&
                   aligned16(wr, wi, hist, x, bx, cw, cb);
  const dim3 grid((B + 15) / 16, blocks);
#define ST(NW, V)                                                             \
  rglru_step_kernel<NW, V><<<grid, 64 * NW, sm, s>>>((u16*)out,               \
      (float*)state, (u16*)hist, (const u16*)x, ldx, (const u16*)bx,          \
      (const u16*)cw, (const u16*)cb, (const u16*)y, ldy, (const u16*)by,     \
      (const u16*)wr, (const float*)br, (const u16*)wi, (const float*)bi,     \
      (const float*)rate, (const i32*)q_start, (const i32*)sslot, B, C, n, taps)
  if (n > 64) { if (vec) ST(8, true); else ST(8, false); }
  else { if (vec) ST(4, true); else ST(4, false); }
#undef ST
  return af_last_err();
}
