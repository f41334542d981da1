// Row kernels of stacks whose sublayers read their normed input plus a short causal convolution of it over time, and whose
// layers hand on a learned average over depth. The residual stream and everything in this file is fp32 except what feeds a GEMM.
//
//     h = x / sqrt(mean x^2 + eps) (1 + w);   g = h + sum_j taps[j] h_(t - K + 1 + j)          (what a sublayer reads)
//     x <- x + f(g);   after a layer's last sublayer X_(i+1) = x and x <- sum_(j <= i+1) c_j X_j    (X_0: the embedding)
//
//   stream_join   one launch per sublayer boundary, one workgroup per token: the finished sublayer's output (a GEMM's, the
//                 shared expert's, the token's routed expert rows with their common weight) joins the stream; behind a layer
//                 the result is kept for later averages and replaced by the average; the next norm's row factor is formed.
//                 Steps of single tokens: the convolution runs here as well (the earlier h are the slot's, none is the
//                 step's) and the slot's ring gets the new h. Steps with portions: the closing sublayer's last h of every
//                 sequence are saved into the ring here, ahead of being overwritten, and canon_conv follows.
//   canon_conv    g for steps with portions: earlier h of the step come from the stream rows and their factors, those of
//                 earlier steps from the slot's ring, those in front of the sequence are zero.
//   poly_norm     a N(z) + b N(z^2) + c N(z^3) + e per row, N dividing the row by its root mean square
//
// The ring of a (slot, sublayer) holds the last K - 1 h, the one of position p in row p mod (K - 1): a portion of any length
// overwrites exactly the rows that fell out of reach, so nothing is shifted, and position 0 needs no clearing (positions in
// front of the sequence are never read).
#include "units.h"
#include "launch.h"

namespace dlia {

constexpr int kCanonThreads = 256;

template <typename OT, int V, int NR>
__global__ __launch_bounds__(kCanonThreads) void stream_join_kernel(
    OT* __restrict__ out, long ldo, float* x, const float* x_in, const float* __restrict__ ya, long ldya,
    const float* __restrict__ yb, long ldyb, const float* __restrict__ ey, const int* __restrict__ pair_row, int top, float ew,
    float* hist, long hist_stride, int navg, const float* __restrict__ coef, const float* __restrict__ nw,
    float* __restrict__ rs, const float* __restrict__ close_w, float* __restrict__ close_carry, const float* __restrict__ taps,
    float* __restrict__ carry, int K, const int* __restrict__ tok_pos, const int* __restrict__ tok_seq, int T, int state_rows, int H,
    float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, units = H / V;
  const int slot = tok_seq[t], pos = tok_pos[t];
  const bool slot_ok = slot >= 0 && slot < state_rows && pos >= 0;
  const long row = (long)t * H;
  Unit<V> r[NR];
  // the closing sublayer's h of this token, if it is among the last K - 1 of its sequence in this step
  const bool keep_h = close_carry && K > 1 && slot_ok && (t + K - 1 >= T || tok_seq[t + K - 1] != slot);
  const float rs_old = keep_h ? rs[t] : 0.f;
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int u = threadIdx.x + k * kCanonThreads;
    if (u >= units) break;
    const int c = u * V;
    r[k] = ldu<V>(x_in + row + c);
    if (keep_h) {
      const Unit<V> w = ldu<V>(close_w + c);
      Unit<V> h;
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] = r[k].v[e] * rs_old * (1.f + w.v[e]);
      stu<V>(close_carry + ((long)slot * (K - 1) + pos % (K - 1)) * H + c, h);
    }
    if (ya) {
      const Unit<V> a = ldu<V>(ya + (long)t * ldya + c);
#pragma unroll
      for (int e = 0; e < V; ++e) r[k].v[e] += a.v[e];
    }
    if (ey || yb) {
      Unit<V> s;
#pragma unroll
      for (int e = 0; e < V; ++e) s.v[e] = 0.f;
      if (ey) {
        for (int i = 0; i < top; ++i) {
          const int er = pair_row[(long)t * top + i];
          if (er < 0) continue;
          const Unit<V> a = ldu<V>(ey + (long)er * H + c);
#pragma unroll
          for (int e = 0; e < V; ++e) s.v[e] += ew * a.v[e];
        }
      }
      if (yb) {
        const Unit<V> b = ldu<V>(yb + (long)t * ldyb + c);
#pragma unroll
        for (int e = 0; e < V; ++e) s.v[e] += b.v[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) r[k].v[e] += s.v[e];
    }
    if (hist) {
      stu<V>(hist + (long)navg * hist_stride + row + c, r[k]);
      Unit<V> s;
#pragma unroll
      for (int e = 0; e < V; ++e) s.v[e] = 0.f;
      for (int j0 = 0; j0 < navg; j0 += 4) {           // (four rows in flight)
        Unit<V> a[4]; float cj[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int jj = min(j0 + j, navg - 1);
          a[j] = ldu<V>(hist + (long)jj * hist_stride + row + c);
          cj[j] = j0 + j < navg ? coef[jj] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (j0 + j < navg)
#pragma unroll
            for (int e = 0; e < V; ++e) s.v[e] += cj[j] * a[j].v[e];
      }
      const float cl = coef[navg];
#pragma unroll
      for (int e = 0; e < V; ++e) r[k].v[e] = s.v[e] + cl * r[k].v[e];
    }
    stu<V>(x + row + c, r[k]);
  }
  if (!nw) return;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    if ((int)threadIdx.x + k * kCanonThreads >= units) break;
#pragma unroll
    for (int e = 0; e < V; ++e) ss += r[k].v[e] * r[k].v[e];
  }
  ss = block_sum(ss, scratch);
  const float f = 1.f / sqrtf(ss / H + eps);
  if (threadIdx.x == 0) rs[t] = f;
  if (!out) return;
  // single-token step: the token's earlier h are all in its slot's ring
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int u = threadIdx.x + k * kCanonThreads;
    if (u >= units) break;
    const int c = u * V;
    const Unit<V> w = ldu<V>(nw + c);
    Unit<V> h, g;
#pragma unroll
    for (int e = 0; e < V; ++e) h.v[e] = r[k].v[e] * f * (1.f + w.v[e]);
    g = h;
    if (taps) {
      Unit<V> s;
#pragma unroll
      for (int e = 0; e < V; ++e) s.v[e] = 0.f;
      for (int j = 0; j < K - 1; ++j) {
        const int p = pos - (K - 1) + j;
        if (p < 0 || !slot_ok) continue;
        const Unit<V> a = ldu<V>(carry + ((long)slot * (K - 1) + p % (K - 1)) * H + c), q = ldu<V>(taps + (long)j * H + c);
#pragma unroll
        for (int e = 0; e < V; ++e) s.v[e] += q.v[e] * a.v[e];
      }
      const Unit<V> q = ldu<V>(taps + (long)(K - 1) * H + c);
#pragma unroll
      for (int e = 0; e < V; ++e) g.v[e] = h.v[e] + (s.v[e] + q.v[e] * h.v[e]);
      if (K > 1 && slot_ok) stu<V>(carry + ((long)slot * (K - 1) + pos % (K - 1)) * H + c, h);
    }
    stu<V>(out + (long)t * ldo + c, g);
  }
}

// A workgroup takes kConvRows consecutive tokens by 256 units of V channels and slides the last h over them in registers: a row is
// read once per tile (and the K - 1 rows in front of it). KT: taps known at compile time, 0: any number, every row read again.
constexpr int kConvRows = 8;

template <typename OT, int V, int KT>
__global__ __launch_bounds__(kCanonThreads) void canon_conv_kernel(
    OT* __restrict__ out, long ldo, const float* __restrict__ x, const float* __restrict__ rs, const float* __restrict__ nw,
    const float* __restrict__ taps, const float* __restrict__ carry, int K, const int* __restrict__ tok_pos,
    const int* __restrict__ tok_seq, int T, int state_rows, int H) {
  const int c = (blockIdx.y * kCanonThreads + threadIdx.x) * V;
  if (c >= H) return;
  Unit<V> w = ldu<V>(nw + c);
#pragma unroll
  for (int e = 0; e < V; ++e) w.v[e] += 1.f;
  auto row_h = [&](int t) {
    Unit<V> h = ldu<V>(x + (long)t * H + c);
    const float f = rs[t];
#pragma unroll
    for (int e = 0; e < V; ++e) h.v[e] = h.v[e] * f * w.v[e];
    return h;
  };
  // h of the token `back` places before token t of the step (position pos of the sequence in `slot`); zeros in front of the sequence
  auto earlier = [&](int t, int back, int slot, int pos) {
    const int p = pos - back;
    Unit<V> h;
#pragma unroll
    for (int e = 0; e < V; ++e) h.v[e] = 0.f;
    if (p < 0) return h;
    if (t - back >= 0 && tok_seq[t - back] == slot && tok_pos[t - back] == p) return row_h(t - back);
    if (slot >= 0 && slot < state_rows) return ldu<V>(carry + ((long)slot * (K - 1) + p % (K - 1)) * H + c);
    return h;
  };
  constexpr int KR = KT > 1 ? KT : 1;
  Unit<V> tap[KR], win[KR];                            // win[j]: the h that meets tap j (the last one is the token's own)
  if constexpr (KT > 0) {
#pragma unroll
    for (int j = 0; j < KT; ++j) tap[j] = ldu<V>(taps + (long)j * H + c);
  }
  const int first = blockIdx.x * kConvRows, t1 = min(T, first + kConvRows);
  int slot_before = -1;
  for (int t = first; t < t1; ++t) {
    const int slot = tok_seq[t], pos = tok_pos[t];
    const Unit<V> h = row_h(t);
    Unit<V> g = h, s;
#pragma unroll
    for (int e = 0; e < V; ++e) s.v[e] = 0.f;
    if constexpr (KT > 0) {
      if (t > first && slot == slot_before) {
#pragma unroll
        for (int j = 0; j + 1 < KT; ++j) win[j] = win[j + 1];
      } else {
#pragma unroll
        for (int j = 0; j + 1 < KT; ++j) win[j] = earlier(t, KT - 1 - j, slot, pos);
      }
      win[KT - 1] = h;
      slot_before = slot;
#pragma unroll
      for (int j = 0; j + 1 < KT; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) s.v[e] += tap[j].v[e] * win[j].v[e];
#pragma unroll
      for (int e = 0; e < V; ++e) g.v[e] = h.v[e] + (s.v[e] + tap[KT - 1].v[e] * h.v[e]);
    } else if (taps) {
      for (int j = 0; j < K - 1; ++j) {
        const Unit<V> a = earlier(t, K - 1 - j, slot, pos), q = ldu<V>(taps + (long)j * H + c);
#pragma unroll
        for (int e = 0; e < V; ++e) s.v[e] += q.v[e] * a.v[e];
      }
      const Unit<V> q = ldu<V>(taps + (long)(K - 1) * H + c);
#pragma unroll
      for (int e = 0; e < V; ++e) g.v[e] = h.v[e] + (s.v[e] + q.v[e] * h.v[e]);
    }
    stu<V>(out + (long)t * ldo + c, g);
  }
}

template <typename OT, int V>
__global__ __launch_bounds__(kCanonThreads) void poly_norm_kernel(OT* __restrict__ out, long ldo, const float* __restrict__ z, long ldz,
                                                                  const float* __restrict__ coef, int F, float eps) {
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  const float* zr = z + t * ldz;
  float s1 = 0.f, s2 = 0.f, s3 = 0.f;
  for (int c = threadIdx.x * V; c < F; c += kCanonThreads * V) {
    const Unit<V> a = ldu<V>(zr + c);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float v = a.v[e], v2 = v * v, v4 = v2 * v2;
      s1 += v2; s2 += v4; s3 += v4 * v2;
    }
  }
  s1 = block_sum(s1, scratch); s2 = block_sum(s2, scratch); s3 = block_sum(s3, scratch);
  const float a1 = coef[0] / sqrtf(s1 / F + eps), a2 = coef[1] / sqrtf(s2 / F + eps), a3 = coef[2] / sqrtf(s3 / F + eps), a0 = coef[3];
  for (int c = threadIdx.x * V; c < F; c += kCanonThreads * V) {
    Unit<V> a = ldu<V>(zr + c);
#pragma unroll
    for (int e = 0; e < V; ++e) { const float v = a.v[e]; a.v[e] = a0 + v * (a1 + v * (a2 + v * a3)); }
    stu<V>(out + t * ldo + c, a);
  }
}

}  // namespace dlia

using namespace dlia;

static bool al16(const void* p) { return (uintptr_t)p % 16 == 0; }

extern "C" int dlia_stream_join_max_width(int vec) { return vec ? 16384 : 4096; }

extern "C" int dlia_stream_join(void* out, int out_f32, long ldo, float* x, const float* x_in, const float* ya, long ldya, const float* yb,
                                long ldyb, const float* ey, const int* pair_row, int top, float ew, float* hist, long hist_stride, int navg,
                                const float* coef, const float* nw, float* rs, const float* close_w, float* close_carry,
                                const float* taps, float* carry, int K, const int* tok_pos, const int* tok_seq, int T, int state_rows,
                                int H, float eps, hipStream_t stream) {
  if (T <= 0) return 0;
  const bool vec = H % 4 == 0 && al16(x) && al16(x_in) && al16(ya) && ldya % 4 == 0 && al16(yb) && ldyb % 4 == 0 && al16(ey) && al16(hist) &&
                   hist_stride % 4 == 0 && al16(nw) && al16(close_w) && al16(close_carry) && al16(taps) && al16(carry) && al16(out) && ldo % 4 == 0;
  const int per = (H / (vec ? 4 : 1) + kCanonThreads - 1) / kCanonThreads;
  if (per > 16) return 1;
#define DLIA_JOIN(OT, V, NR)                                                                                                       \
  hipLaunchKernelGGL((stream_join_kernel<OT, V, NR>), dim3(T), dim3(kCanonThreads), 0, stream, (OT*)out, ldo, x, x_in, ya, ldya, yb, ldyb, \
                     ey, pair_row, top, ew, hist, hist_stride, navg, coef, nw, rs, close_w, close_carry, taps, carry, K, tok_pos, tok_seq, \
                     T, state_rows, H, eps)
#define DLIA_JOIN_NR(OT, V)                                                                                         \
  do {                                                                                                              \
    if (per <= 1) DLIA_JOIN(OT, V, 1); else if (per <= 2) DLIA_JOIN(OT, V, 2); else if (per <= 4) DLIA_JOIN(OT, V, 4); \
    else if (per <= 8) DLIA_JOIN(OT, V, 8); else DLIA_JOIN(OT, V, 16);                                              \
  } while (0)
  if (out && !out_f32) { if (vec) DLIA_JOIN_NR(bf16, 4); else DLIA_JOIN_NR(bf16, 1); }
  else { if (vec) DLIA_JOIN_NR(float, 4); else DLIA_JOIN_NR(float, 1); }
#undef DLIA_JOIN_NR
#undef DLIA_JOIN
  return 0;
}

extern "C" void dlia_canon_conv(void* out, int out_f32, long ldo, const float* x, const float* rs, const float* nw, const float* taps,
                                const float* carry, int K, const int* tok_pos, const int* tok_seq, int T, int state_rows, int H,
                                hipStream_t stream) {
  if (T <= 0) return;
  const bool vec = H % 4 == 0 && al16(x) && al16(nw) && al16(taps) && al16(carry) && al16(out) && ldo % 4 == 0;
  const int per = kCanonThreads * (vec ? 4 : 1);
  const dim3 grid((T + kConvRows - 1) / kConvRows, (H + per - 1) / per);
#define DLIA_CONV(OT, V, KT)                                                                                                        \
  hipLaunchKernelGGL((canon_conv_kernel<OT, V, KT>), grid, dim3(kCanonThreads), 0, stream, (OT*)out, ldo, x, rs, nw, taps, carry, K, \
                     tok_pos, tok_seq, T, state_rows, H)
#define DLIA_CONV_K(OT)                                                                                       \
  do {                                                                                                        \
    if (!vec) DLIA_CONV(OT, 1, 0); else if (taps && K == 2) DLIA_CONV(OT, 4, 2); else if (taps && K == 3) DLIA_CONV(OT, 4, 3); \
    else if (taps && K == 4) DLIA_CONV(OT, 4, 4); else DLIA_CONV(OT, 4, 0);                                   \
  } while (0)
  if (out_f32) DLIA_CONV_K(float); else DLIA_CONV_K(bf16);
#undef DLIA_CONV_K
#undef DLIA_CONV
}

extern "C" void dlia_poly_norm(void* out, int out_f32, long ldo, const float* z, long ldz, const float* coef, int T, int F, float eps,
                               hipStream_t stream) {
  if (T <= 0) return;
  const bool vec = F % 4 == 0 && al16(z) && ldz % 4 == 0 && al16(out) && ldo % 4 == 0;
#define DLIA_POLY(OT, V) \
  hipLaunchKernelGGL((poly_norm_kernel<OT, V>), dim3(T), dim3(kCanonThreads), 0, stream, (OT*)out, ldo, z, ldz, coef, F, eps)
  if (out_f32) { if (vec) DLIA_POLY(float, 4); else DLIA_POLY(float, 1); }
  else { if (vec) DLIA_POLY(bf16, 4); else DLIA_POLY(bf16, 1); }
#undef DLIA_POLY
}
