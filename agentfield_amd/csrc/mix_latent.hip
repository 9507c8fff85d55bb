// Row steps of latent attention: latent norm, rotary positions, cache append
// and query assembly in front of the attention kernel, gated head outputs
// behind it.
//
// Storage dtype S is bf16 (raw u16) or fp32; the norm, the rotation and the
// gate are fp32.
#include "mix_rows.h"

namespace {

// One workgroup per row.  The down projection's row holds the latent (first
// R values) and one rotary key part (rd values); the latent is RMS-normed
// with a plain weight, the key part rotated, and [latent | key part] goes to
// the key pages [P, 1, page, R + rd] at `slot` (without dkv the row only has
// queries: its layer reads another layer's pages).  The attention query of
// head h is [q in latent space (R, already in place) | rotate(q[t, h,
// dim:dim+rd])]: the kernel fills the rotary slices of qf [T, H, R + rd].
// Rotation: pair i < rot/2 turns by the row's table entry, `inter` pairs
// element 2i with 2i+1, otherwise i with i + rot/2; elements past rot pass.
//
// V4: a work item is two neighbouring pairs (four elements: one run of four,
// or two runs of two), for rot a multiple of 4 and aligned rows.
template <typename S, bool V4>
__global__ void __launch_bounds__(256) latent_prep_kernel(
    S* __restrict__ qf, S* __restrict__ kc, const S* __restrict__ q, i64 ldq,
    const S* __restrict__ dkv, i64 lddkv, const S* __restrict__ normw,
    const float* __restrict__ tab, const i64* __restrict__ slots, float eps,
    int H, int dim, int rd, int R, int rot, int inter) {
  __shared__ float red[4];
  extern __shared__ float cs[];              // [rot/2] cos, [rot/2] sin
  const int t = blockIdx.x;
  const int half = rot / 2;
  for (int i = threadIdx.x; i < rot; i += 256) cs[i] = tab[(size_t)t * rot + i];
  const int dkc = R + rd;
  const S* dr = dkv ? dkv + (size_t)t * lddkv : nullptr;
  float ss = 0.f;
  if (dr) {
    if constexpr (V4) {
      for (int i = threadIdx.x * 4; i < R; i += 1024) {
        float v[4];
        ldv<S, 4>(dr + i, v);
        ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
      }
    } else {
      for (int i = threadIdx.x; i < R; i += 256) {
        const float v = ldf<S>(dr + i);
        ss += v * v;
      }
    }
    ss = wave_sum_f32(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
  }
  __syncthreads();                           // table and partial sums
  const i64 sl = slots[t];
  S* kr = (dr && sl >= 0) ? kc + (size_t)sl * dkc : nullptr;  // one K/V head
  if (kr) {
    const float rinv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)R + eps);
    if constexpr (V4) {
      for (int i = threadIdx.x * 4; i < R; i += 1024) {
        float v[4], w[4];
        ldv<S, 4>(dr + i, v);
        ldv<S, 4>(normw + i, w);
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] *= rinv * w[j];
        stv<S, 4>(kr + i, v);
      }
    } else {
      for (int i = threadIdx.x; i < R; i += 256)
        stf<S>(kr + i, ldf<S>(dr + i) * rinv * ldf<S>(normw + i));
    }
  }
  // rotary slices: unit 0 is the key part (when there is one), the others
  // the heads
  const int dq = dim + rd;
  const int k0 = kr ? 0 : 1;
  const int units = H + 1 - k0;
  auto src_of = [&](int u) {
    return u == 0 ? dr + R : q + (size_t)t * ldq + (size_t)(u - 1) * dq + dim;
  };
  auto dst_of = [&](int u) {
    return u == 0 ? kr + R : qf + ((size_t)t * H + u - 1) * dkc + R;
  };
  if constexpr (V4) {
    const int per = rd / 4, rper = rot / 4;
    for (int i = threadIdx.x; i < units * per; i += 256) {
      const int u = i / per + k0, w = i % per;
      const S* src = src_of(u);
      S* dst = dst_of(u);
      if (w >= rper) {                       // passes unchanged
        float v[4];
        ldv<S, 4>(src + w * 4, v);
        stv<S, 4>(dst + w * 4, v);
      } else if (inter) {
        float v[4], o[4];
        ldv<S, 4>(src + w * 4, v);
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const float c = cs[w * 2 + j], s = cs[half + w * 2 + j];
          o[2 * j] = v[2 * j] * c - v[2 * j + 1] * s;
          o[2 * j + 1] = v[2 * j + 1] * c + v[2 * j] * s;
        }
        stv<S, 4>(dst + w * 4, o);
      } else {
        float a[2], b[2];
        ld2<S, true>(src + w * 2, a[0], a[1]);
        ld2<S, true>(src + half + w * 2, b[0], b[1]);
        const float c0 = cs[w * 2], c1 = cs[w * 2 + 1];
        const float s0 = cs[half + w * 2], s1 = cs[half + w * 2 + 1];
        st2<S, true>(dst + w * 2, a[0] * c0 - b[0] * s0, a[1] * c1 - b[1] * s1);
        st2<S, true>(dst + half + w * 2, b[0] * c0 + a[0] * s0, b[1] * c1 + a[1] * s1);
      }
    }
  } else {
    for (int i = threadIdx.x; i < units * rd; i += 256) {
      const int u = i / rd + k0, k = i % rd;
      const S* src = src_of(u);
      float v = ldf<S>(src + k);
      if (k < rot) {
        const int pr = inter ? k >> 1 : (k < half ? k : k - half);
        const int mate = inter ? k ^ 1 : (k < half ? k + half : k - half);
        const bool second = inter ? (k & 1) : k >= half;
        const float o = ldf<S>(src + mate);
        v = v * cs[pr] + o * (second ? cs[half + pr] : -cs[half + pr]);
      }
      stf<S>(dst_of(u) + k, v);
    }
  }
}

// out[t, h*dv + d] = o[h, t, d] * sigmoid(gate): head-major per-head results
// back to token rows, times the output gate: one logit per element, g[t,
// h*dv + d], or (HEAD) one per head, g[t, h].
template <typename S, int V, bool HEAD>
__global__ void __launch_bounds__(256) gate_heads_kernel(
    S* __restrict__ out, const S* __restrict__ o, const S* __restrict__ g,
    i64 ldg, int T, int H, int dv) {
  const int per = dv / V;
  const i64 total = (i64)T * H * per;
  for (i64 i = (i64)blockIdx.x * 256 + threadIdx.x; i < total;
       i += (i64)gridDim.x * 256) {
    const int d = (int)(i % per) * V;
    const int h = (int)((i / per) % H);
    const i64 t = i / ((i64)per * H);
    float gv[4], ov[4];
    if constexpr (HEAD) gv[0] = gv[1] = gv[2] = gv[3] = ldf<S>(g + t * ldg + h);
    else ldv<S, V>(g + t * ldg + (i64)h * dv + d, gv);
    ldv<S, V>(o + ((i64)h * T + t) * dv + d, ov);
#pragma unroll
    for (int j = 0; j < V; ++j) ov[j] = ov[j] / (1.0f + expf(-gv[j]));
    stv<S, V>(out + (t * H + h) * dv + d, ov);
  }
}

template <typename S>
int launch_latent_prep(void* qf, void* kc, const void* q, i64 ldq,
                       const void* dkv, i64 lddkv, const void* normw,
                       const void* tab, const void* slots, float eps, int T,
                       int H, int dim, int rd, int R, int rot, int inter,
                       hipStream_t s) {
  const size_t sm = (size_t)(rot > 0 ? rot : 1) * sizeof(float);
  const bool v4 = R % 4 == 0 && rd % 4 == 0 && rot % 4 == 0 && dim % 4 == 0 &&
                  ldq % 4 == 0 && lddkv % 4 == 0 &&
                  aligned16(qf, kc, q, dkv, normw);
#define LP(V4)                                                               \
  latent_prep_kernel<S, V4><<<T, 256, sm, s>>>((S*)qf, (S*)kc, (const S*)q,  \
      ldq, (const S*)dkv, lddkv, (const S*)normw, (const float*)tab,         \
      (const i64*)slots, eps, H, dim, rd, R, rot, inter)
  if (v4) LP(true); else LP(false);
#undef LP
  return af_last_err();
}

}  // namespace

// tab [T, rot] fp32: the rows' cos | sin (afm_rotary_table).  dkv null: no
// key row is written (then kc and normw may be null too).
AF_EXPORT int afm_latent_prep(void* qf, void* kc, const void* q, i64 ldq,
                              const void* dkv, i64 lddkv, const void* normw,
                              const void* tab, const void* slots, float eps,
                              int T, int H, int dim, int rd, int R, int rot,
                              int inter, int dt, void* stream) {
  if (T == 0) return 0;
  if (rot < 0 || rot > rd || (rot & 1) || (rot && !tab)) return 9003;
  if (dkv && (!kc || !normw)) return 9003;
  hipStream_t s = (hipStream_t)stream;
  if (dt == 0)
    return launch_latent_prep<u16>(qf, kc, q, ldq, dkv, lddkv, normw, tab,
                                   slots, eps, T, H, dim, rd, R, rot, inter, s);
  if (dt == 1)
    return launch_latent_prep<float>(qf, kc, q, ldq, dkv, lddkv, normw, tab,
                                     slots, eps, T, H, dim, rd, R, rot, inter, s);
  return 9002;
}

AF_EXPORT int afm_gate_heads(void* out, const void* o, const void* g, i64 ldg,
                             int T, int H, int dv, int per_head, int dt,
                             void* stream) {
  if (T == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = dv % 4 == 0 && aligned16(out, o) &&
                   (per_head || (ldg % 4 == 0 && aligned16(g)));
  const i64 total = (i64)T * H * (vec ? dv / 4 : dv);
  const int grid = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
#define GH(S, V, HD)                                                          \
  gate_heads_kernel<S, V, HD><<<grid, 256, 0, s>>>((S*)out, (const S*)o,      \
                                                   (const S*)g, ldg, T, H, dv)
#define GHV(S, V) do { if (per_head) GH(S, V, true); else GH(S, V, false); } while (0)
  if (dt == 0) { if (vec) GHV(u16, 4); else GHV(u16, 1); }
  else if (dt == 1) { if (vec) GHV(float, 4); else GHV(float, 1); }
  else return 9002;
#undef GHV
#undef GH
  return af_last_err();
}
