// Linear attention with decays: per head a state S [d, dv] in the sequence's slot,
//     S <- diag(a_t) S + k_t v_t^T,   o_t = S^T (c q_t),   out = rms(o) w * silu(g),
// a_t one number per head from the config, or one per key channel, sigmoid(z)^(1 / tau) with z = W2 (low-rank projection of the
// input) + b. q, k, v, g and the low-rank projection are columns of the input GEMM's fp32 output. Everything here is fp32: the
// products run on the 16x16x4 fp32 MFMA (true 32-bit), in the bf16 mode as well.
//
// Steps of single tokens (decoding): one workgroup per (sequence, head) streams the head's state once (read, update, write back)
// with the read-out, the per-head norm and the gate in the same launch.
//
// Steps with portions are worked in chunks of 64 tokens per sequence, in three launches:
//   local   per (sequence, head, chunk, 64 key channels): log decays and their running sums inside each quarter of the chunk, what
//           the chunk adds to a state, sum_t exp(G_end - G_t) k_t v_t^T (G the running sum of the log decays over the chunk)
//   carry   per (sequence, head), element by element: the chunks' additions become the states in front of the chunks, the slot
//           gets the last one
//   out     per (sequence, head, chunk): exp(G_i) q_i . S_before + sum_(j <= i) (sum_c q_ic k_jc exp(G_ic - G_jc)) v_j, the norm
//           over the head's values, the gate
// A decay per channel cannot be taken out of the score product as exp(G_i) exp(-G_j) (the second factor overflows), so each
// quarter of 16 tokens keeps its own references: q carries exp(G_i - G_start of i's quarter), k carries exp(G_end of j's quarter -
// G_j), both at most one, and the score tile of two quarters gets the factor between the two references, which is at most one for
// different quarters. Inside a quarter that factor is exp(-(the quarter's sum)): where it grows large (a sum below
// -60 in log2), the tile's pairs are summed one by one from exp(G_i - G_j) itself.
// Log decays are kept in units of log2, so that every factor is one hardware exp2.
// A portion may start and end anywhere: chunks are counted from the portion's first token, and the split only changes rounding.
#include "units.h"
#include "launch.h"

namespace dlia {

constexpr int kLaChunk = 64;
constexpr int kLaQuarter = 16;
constexpr int kLaCh = 64;              // key channels at a time
constexpr int kLaVals = 128;           // value columns at a time in `local`
constexpr float kLaFar = -60.f;        // (in log2)
constexpr float kLaLog2e = 1.4426950408889634f;

struct LaArgs {
  void* out; long ldo;
  const float* z; long ldz;
  float* state;
  const float* head_decay;             // [2][H]: decay, log2 of it; null: a decay per channel
  const float* a2t; const float* a_b;  // [rank][H d], [H d]
  const float* norm_w;                 // [dv] or null
  float* ws_state; float* ws_dec; float* g;
  const int* q_start; const int* ctx; const int* slots;
  int H, d, dv, rank, state_rows, nblk;
  int col_q, col_k, col_v, col_g, col_a;
  float qscale, inv_tau, eps;
  int vec;                             // value columns of z come in aligned groups of four
};

// base^n for log2(base) = l2 (minus infinity for base 0)
__device__ __forceinline__ float pow_n(int n, float l2) { return n == 0 ? 1.f : exp2f((float)n * l2); }
__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float la_gate(float g) { return g / (1.f + expf(-g)); }
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// ---- single tokens --------------------------------------------------------------------------------------------------
template <typename OT, int V>
__global__ __launch_bounds__(256) void la_decode_kernel(LaArgs p) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float scratch[16];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int t = p.q_start[b], n = p.q_start[b + 1] - t, slot = p.slots[b];
  if (n != 1 || slot < 0 || slot >= p.state_rows) return;
  const bool fresh = p.ctx[b] <= 0;
  const int d = p.d, dv = p.dv;
  const int units = (dv + V - 1) / V, CT = min(units, 256), RG = 256 / CT, ct = tid % CT, rg = tid / CT;
  float* qv = lds; float* kv = qv + d; float* av = kv + d;
  float* po = lds + (3 * d + 3) / 4 * 4;                     // [RG][dv]
  const float* zr = p.z + (long)t * p.ldz;
  for (int i = tid; i < d; i += 256) {
    qv[i] = zr[p.col_q + h * d + i] * p.qscale;
    kv[i] = zr[p.col_k + h * d + i];
    float a;
    if (p.head_decay) a = p.head_decay[h];
    else {
      float s = p.a_b[h * d + i];
      for (int r = 0; r < p.rank; ++r) s += zr[p.col_a + r] * p.a2t[(long)r * p.H * d + h * d + i];
      a = expf(log_sigmoid(s) * p.inv_tau);
    }
    av[i] = a;
  }
  __syncthreads();
  float* S = p.state + ((long)slot * p.H + h) * (long)d * dv;
  constexpr int U = 8;                                       // rows in flight
  if (rg < RG) {
    for (int u = ct; u < units; u += CT) {
      const int col = u * V;
      const Unit<V> v = ldu<V>(zr + p.col_v + (long)h * dv + col);
      Unit<V> acc;
#pragma unroll
      for (int e = 0; e < V; ++e) acc.v[e] = 0.f;
      for (int r0 = rg; r0 < d; r0 += RG * U) {
        Unit<V> s[U];
#pragma unroll
        for (int i = 0; i < U; ++i) {
          const int r = r0 + i * RG;
          if (r < d && !fresh) s[i] = ldu<V>(S + (long)r * dv + col);
          else {
#pragma unroll
            for (int e = 0; e < V; ++e) s[i].v[e] = 0.f;
          }
        }
#pragma unroll
        for (int i = 0; i < U; ++i) {
          const int r = r0 + i * RG;
          if (r >= d) break;
          const float a = av[r], k = kv[r], q = qv[r];
#pragma unroll
          for (int e = 0; e < V; ++e) {
            s[i].v[e] = a * s[i].v[e] + k * v.v[e];
            acc.v[e] += q * s[i].v[e];
          }
          stu<V>(S + (long)r * dv + col, s[i]);
        }
      }
      stu<V>(po + rg * dv + col, acc);
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < dv; c += 256) {
    float o = 0.f;
    for (int i = 0; i < RG; ++i) o += po[i * dv + c];
    po[c] = o;                                               // (column c belongs to this thread alone)
    ss += o * o;
  }
  ss = block_sum(ss, scratch);
  const float r = 1.f / sqrtf(ss / dv + p.eps);
  OT* orow = (OT*)p.out + (long)t * p.ldo + (long)h * dv;
  for (int c = tid; c < dv; c += 256)
    orow[c] = (OT)(po[c] * r * (p.norm_w ? p.norm_w[c] : 1.f) * la_gate(zr[p.col_g + (long)h * dv + c]));
}

// ---- portions: what a chunk adds to a state ---------------------------------------------------------------------------
__device__ __forceinline__ long la_chunk_row(int t0, int b) { return t0 / kLaChunk + b; }     // (rows of different sequences never meet)

__global__ __launch_bounds__(256) void la_local_kernel(LaArgs p) {
  constexpr int KST = kLaCh + 16, VST = kLaVals + 16;        // (rows 16 banks apart: the four k-rows of a fragment do not collide)
  __shared__ __attribute__((aligned(16))) float ks[kLaChunk * KST];
  __shared__ __attribute__((aligned(16))) float vs[kLaChunk * VST];
  __shared__ float tot[4][kLaCh];
  const int h = blockIdx.x, b = blockIdx.y, chunk = blockIdx.z / p.nblk, db = blockIdx.z % p.nblk;
  const int t0 = p.q_start[b], n = p.q_start[b + 1] - t0, slot = p.slots[b];
  const int nt = min(kLaChunk, n - chunk * kLaChunk);
  if (nt <= 0 || slot < 0 || slot >= p.state_rows) return;   // (whole workgroup)
  const int tid = threadIdx.x, d = p.d, dv = p.dv;
  const long tq = (long)t0 + chunk * kLaChunk, crow = la_chunk_row(t0, b) + chunk;
  const int c = tid & 63, qt = tid >> 6, ch = db * kLaCh + c;
  const bool ok = ch < d;
  const float* zq = p.z + tq * p.ldz;
  float f[kLaQuarter];                                       // factor of this thread's 16 tokens in its channel
  if (p.head_decay) {
    const float l2 = p.head_decay[p.H + h];
#pragma unroll
    for (int i = 0; i < kLaQuarter; ++i) { const int row = qt * kLaQuarter + i; f[i] = row < nt ? pow_n(nt - 1 - row, l2) : 0.f; }
  } else {
    const long ac = (long)h * d + (ok ? ch : 0);
    const float bias = p.a_b[ac];
#pragma unroll
    for (int i = 0; i < kLaQuarter; ++i) f[i] = bias;
    // the chunk's low-rank projections go through LDS (the values' buffer, not in use yet)
    const bool staged = p.rank <= VST;
    if (staged) {
      for (int i = tid; i < nt * p.rank; i += 256) vs[i] = zq[(long)(i / p.rank) * p.ldz + p.col_a + i % p.rank];
      __syncthreads();
    }
    const float* low = staged ? vs : zq + p.col_a;
    const long lrow = staged ? p.rank : p.ldz;
    for (int r0 = 0; r0 < p.rank; r0 += 4) {
      float w[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) w[u] = r0 + u < p.rank ? p.a2t[(long)(r0 + u) * p.H * d + ac] : 0.f;
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (r0 + u < p.rank) {
#pragma unroll
          for (int i = 0; i < kLaQuarter; ++i) f[i] += low[min(qt * kLaQuarter + i, nt - 1) * lrow + r0 + u] * w[u];
        }
    }
    const float unit = p.inv_tau * kLaLog2e;
    float run = 0.f;
#pragma unroll
    for (int i = 0; i < kLaQuarter; ++i) {
      const int row = qt * kLaQuarter + i;
      if (row < nt) run += log_sigmoid(f[i]) * unit;
      f[i] = run;
      if (ok && row < nt) p.g[(tq + row) * p.H * d + ac] = run;
    }
    tot[qt][c] = run;
    __syncthreads();
    float rest = run;
    for (int j = qt + 1; j < 4; ++j) rest += tot[j][c];
    if (qt == 0 && ok) p.ws_dec[crow * p.H * d + ac] = ex2(rest);
#pragma unroll
    for (int i = 0; i < kLaQuarter; ++i) f[i] = qt * kLaQuarter + i < nt ? ex2(rest - f[i]) : 0.f;
  }
#pragma unroll
  for (int i = 0; i < kLaQuarter; ++i) {
    const int row = qt * kLaQuarter + i;
    ks[row * KST + c] = ok && row < nt ? zq[(long)row * p.ldz + p.col_k + h * d + ch] * f[i] : 0.f;
  }
  const int wave = tid >> 6, lane = tid & 63, r16 = lane & 15, kq = lane >> 4;
  float* dst = p.ws_state + (crow * p.H + h) * (long)d * dv;
  for (int v0 = 0; v0 < dv; v0 += kLaVals) {
    __syncthreads();
    {
      // every thread: four neighbouring columns of every eighth token, all loads in flight before the first is parked
      const int cc = (tid & 31) * 4, r8 = tid >> 5;
      const float* src = zq + p.col_v + (long)h * dv + v0 + cc;
      f32x4 v[kLaChunk / 8];
#pragma unroll
      for (int i = 0; i < kLaChunk / 8; ++i) {
        const int row = r8 + i * 8;
        v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (row < nt) {
          if (p.vec) { if (v0 + cc < dv) v[i] = *reinterpret_cast<const f32x4*>(src + (long)row * p.ldz); }
          else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (v0 + cc + e < dv) v[i][e] = src[(long)row * p.ldz + e];
          }
        }
      }
#pragma unroll
      for (int i = 0; i < kLaChunk / 8; ++i) *reinterpret_cast<f32x4*>(vs + (r8 + i * 8) * VST + cc) = v[i];
    }
    __syncthreads();
    if (db * kLaCh + wave * 16 >= d) continue;               // (no barrier until the next round's, which every wave reaches)
    float a[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) a[s] = ks[(s * 4 + kq) * KST + wave * 16 + r16];
#pragma unroll
    for (int ct = 0; ct < kLaVals / 16; ++ct) {
      if (v0 + ct * 16 >= dv) break;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 16; ++s)
        if (s * 4 < nt) acc = mfma4(a[s], vs[(s * 4 + kq) * VST + ct * 16 + r16], acc);
      const int col = v0 + ct * 16 + r16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = db * kLaCh + wave * 16 + kq * 4 + r;
        if (row < d && col < dv) dst[(long)row * dv + col] = acc[r];
      }
    }
  }
}

// ---- portions: the states in front of the chunks ------------------------------------------------------------------------
template <int V>
__global__ __launch_bounds__(256) void la_carry_kernel(LaArgs p) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int t0 = p.q_start[b], n = p.q_start[b + 1] - t0, slot = p.slots[b];
  if (n <= 0 || slot < 0 || slot >= p.state_rows) return;
  const long e = ((long)blockIdx.x * 256 + threadIdx.x) * V, size = (long)p.d * p.dv;
  if (e >= size) return;
  const int row = (int)(e / p.dv), chunks = (n + kLaChunk - 1) / kLaChunk;
  float* w = p.ws_state + (la_chunk_row(t0, b) * p.H + h) * size + e;
  const long step = (long)p.H * size, dstep = (long)p.H * p.d;
  const float* dec = p.head_decay ? nullptr : p.ws_dec + la_chunk_row(t0, b) * dstep + (long)h * p.d + row;
  const float l2 = p.head_decay ? p.head_decay[p.H + h] : 0.f, full = p.head_decay ? pow_n(kLaChunk, l2) : 0.f;
  float* S = p.state + ((long)slot * p.H + h) * size + e;
  Unit<V> s;
  if (p.ctx[b] > 0) s = ldu<V>(S);
  else {
#pragma unroll
    for (int i = 0; i < V; ++i) s.v[i] = 0.f;
  }
  constexpr int D = 4;                                       // chunks in flight
  for (int c0 = 0; c0 < chunks; c0 += D) {
    Unit<V> a[D]; float f[D];
#pragma unroll
    for (int i = 0; i < D; ++i)
      if (c0 + i < chunks) {
        a[i] = ldu<V>(w + (c0 + i) * step);
        f[i] = dec ? dec[(c0 + i) * dstep] : (c0 + i + 1 < chunks ? full : pow_n(n - (c0 + i) * kLaChunk, l2));
      }
#pragma unroll
    for (int i = 0; i < D; ++i)
      if (c0 + i < chunks) {
        stu<V>(w + (c0 + i) * step, s);
#pragma unroll
        for (int k = 0; k < V; ++k) s.v[k] = f[i] * s.v[k] + a[i].v[k];
      }
  }
  stu<V>(S, s);
}

// ---- portions: read-outs ------------------------------------------------------------------------------------------------
// Eight waves. Score tiles (query quarter I, key quarter J <= I): wave w forms tiles w and w + 8 of the ten. Values: wave w owns
// the column tiles w, w + 8, ... of 16 columns for all 64 tokens.
template <typename OT, int NCT, bool HEAD>
__global__ __launch_bounds__(512) void la_out_kernel(LaArgs p) {
  constexpr int ST = kLaCh + 4;
  __shared__ __attribute__((aligned(16))) float qs[kLaChunk * ST];
  __shared__ __attribute__((aligned(16))) float ks[kLaChunk * ST];
  __shared__ __attribute__((aligned(16))) float ps[kLaChunk * ST];
  __shared__ float tot[4][kLaCh];
  __shared__ float red[8][kLaChunk];
  const int h = blockIdx.x, b = blockIdx.y, chunk = blockIdx.z;
  const int t0 = p.q_start[b], n = p.q_start[b + 1] - t0, slot = p.slots[b];
  const int nt = min(kLaChunk, n - chunk * kLaChunk);
  if (nt <= 0 || slot < 0 || slot >= p.state_rows) return;   // (whole workgroup)
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, kq = lane >> 4;
  const int d = p.d, dv = p.dv, mt = (nt + 15) / 16;
  const long tq = (long)t0 + chunk * kLaChunk;
  const float* zq = p.z + tq * p.ldz;
  const float* S = p.ws_state + ((la_chunk_row(t0, b) + chunk) * p.H + h) * (long)d * dv;
  const float l2 = HEAD ? p.head_decay[p.H + h] : 0.f;
  f32x4 acc[4][NCT], sc[2];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int u = 0; u < NCT; ++u) acc[i][u] = f32x4{0.f, 0.f, 0.f, 0.f};
  sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
  // tile number -> (I, J): row by row of the lower triangle
  auto tile_of = [](int x, int& I, int& J) { I = x >= 6 ? 3 : x >= 3 ? 2 : x >= 1 ? 1 : 0; J = x - I * (I + 1) / 2; };
  for (int db = 0; db * kLaCh < d; ++db) {
    // the state's fragments of this wave's columns are asked for first
    float sreg[NCT][16];
#pragma unroll
    for (int u = 0; u < NCT; ++u) {
      const int col = (wave + 8 * u) * 16 + r16;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int ch = db * kLaCh + (i >> 2) * 16 + kq * 4 + (i & 3);
        sreg[u][i] = ch < d && col < dv ? S[(long)ch * dv + col] : 0.f;
      }
    }
    __syncthreads();
    {
      const int c = tid & 63, r8 = tid >> 6, ch = db * kLaCh + c, qt = r8 >> 1;
      const bool ok = ch < d;
      float total = 0.f;
      const long gc = (long)h * d + ch;
      if constexpr (!HEAD) {
        if (ok && qt * kLaQuarter < nt) total = p.g[(tq + min(qt * kLaQuarter + kLaQuarter - 1, nt - 1)) * p.H * d + gc];
        if (!(r8 & 1)) tot[qt][c] = total;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int row = r8 * 8 + i;
        float q = 0.f, k = 0.f;
        if (ok && row < nt) {
          q = zq[(long)row * p.ldz + p.col_q + h * d + ch] * p.qscale;
          k = zq[(long)row * p.ldz + p.col_k + h * d + ch];
          if constexpr (!HEAD) {
            const float g = p.g[(tq + row) * p.H * d + gc];
            q *= ex2(g);
            k *= ex2(total - g);
          }
        }
        qs[row * ST + c] = q;
        ks[row * ST + c] = k;
      }
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int x = wave + 8 * s;
      int I, J;
      tile_of(x, I, J);
      if (x >= 10 || I >= mt) continue;
      if constexpr (!HEAD) {
        if (I == J && __any(tot[I][lane] < kLaFar)) {
          // decays too strong for one reference: pair by pair
          const int j = J * 16 + r16;
          for (int c = 0; c < kLaCh && db * kLaCh + c < d; ++c) {
            const int ch = db * kLaCh + c;
            if (j >= nt) break;
            const float k = zq[(long)j * p.ldz + p.col_k + h * d + ch], gj = p.g[(tq + j) * p.H * d + (long)h * d + ch];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int i = I * 16 + kq * 4 + r;
              if (i >= j && i < nt)
                sc[s][r] += zq[(long)i * p.ldz + p.col_q + h * d + ch] * p.qscale * k * ex2(p.g[(tq + i) * p.H * d + (long)h * d + ch] - gj);
            }
          }
          continue;
        }
      }
#pragma unroll
      for (int k4 = 0; k4 < 4; ++k4) {
        const int c = k4 * 16 + kq * 4;
        f32x4 qa = *reinterpret_cast<const f32x4*>(qs + (I * 16 + r16) * ST + c);
        const f32x4 kb = *reinterpret_cast<const f32x4*>(ks + (J * 16 + r16) * ST + c);
        if constexpr (!HEAD) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float f = I == J ? -tot[I][c + e] : 0.f;
            for (int m = J + 1; m < I; ++m) f += tot[m][c + e];
            qa[e] *= ex2(f);
          }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) sc[s] = mfma4(qa[e], kb[e], sc[s]);
      }
    }
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      if (I >= mt || wave * 16 >= dv) break;
#pragma unroll
      for (int k4 = 0; k4 < 4; ++k4) {
        const int c = k4 * 16 + kq * 4;
        f32x4 qa = *reinterpret_cast<const f32x4*>(qs + (I * 16 + r16) * ST + c);
        if constexpr (!HEAD) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float f = 0.f;
#pragma unroll
            for (int m = 0; m < I; ++m) f += tot[m][c + e];
            if (I > 0) qa[e] *= ex2(f);
          }
        }
#pragma unroll
        for (int u = 0; u < NCT; ++u)
#pragma unroll
          for (int e = 0; e < 4; ++e) acc[I][u] = mfma4(qa[e], sreg[u][k4 * 4 + e], acc[I][u]);
      }
    }
  }
  // the values this wave multiplies
  float vreg[NCT][16];
#pragma unroll
  for (int u = 0; u < NCT; ++u) {
    const int col = (wave + 8 * u) * 16 + r16;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = (i >> 2) * 16 + kq * 4 + (i & 3);
      vreg[u][i] = t < nt && col < dv ? zq[(long)t * p.ldz + p.col_v + (long)h * dv + col] : 0.f;
    }
  }
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const int x = wave + 8 * s;
    int I, J;
    tile_of(x, I, J);
    if (x >= 10) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = I * 16 + kq * 4 + r, j = J * 16 + r16;
      float v = sc[s][r];
      if constexpr (HEAD) v *= j <= i ? pow_n(i - j, l2) : 0.f;
      ps[i * ST + j] = j <= i ? v : 0.f;
    }
  }
  __syncthreads();
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    if constexpr (HEAD) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float f = pow_n(I * 16 + kq * 4 + r + 1, l2);
#pragma unroll
        for (int u = 0; u < NCT; ++u) acc[I][u][r] *= f;
      }
    }
    if (I < mt && wave * 16 < dv) {
#pragma unroll
      for (int k4 = 0; k4 <= I; ++k4) {
        const f32x4 pa = *reinterpret_cast<const f32x4*>(ps + (I * 16 + r16) * ST + k4 * 16 + kq * 4);
#pragma unroll
        for (int u = 0; u < NCT; ++u)
#pragma unroll
          for (int e = 0; e < 4; ++e) acc[I][u] = mfma4(pa[e], vreg[u][k4 * 4 + e], acc[I][u]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float ss = 0.f;
#pragma unroll
      for (int u = 0; u < NCT; ++u) ss += acc[I][u][r] * acc[I][u][r];      // (columns beyond dv are zero)
      ss = group_sum<16>(ss);
      if (r16 == 0) red[wave][I * 16 + kq * 4 + r] = ss;
    }
  }
  __syncthreads();
#pragma unroll
  for (int I = 0; I < 4; ++I)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = I * 16 + kq * 4 + r;
      if (row >= nt) continue;
      float ss = 0.f;
#pragma unroll
      for (int w = 0; w < 8; ++w) ss += red[w][row];
      const float f = 1.f / sqrtf(ss / dv + p.eps);
      OT* orow = (OT*)p.out + (tq + row) * p.ldo + (long)h * dv;
#pragma unroll
      for (int u = 0; u < NCT; ++u) {
        const int col = (wave + 8 * u) * 16 + r16;
        if (col < dv)
          orow[col] = (OT)(acc[I][u][r] * f * (p.norm_w ? p.norm_w[col] : 1.f) * la_gate(zq[(long)row * p.ldz + p.col_g + (long)h * dv + col]));
      }
    }
}

}  // namespace dlia

using namespace dlia;

// Floats of the workspace of a step of `rows` tokens in B sequences: the chunks' states, their decays and the running log decays.
extern "C" long dlia_linear_attention_ws_floats(int rows, int B, int H, int d, int dv, int per_channel) {
  const long chunks = (long)rows / kLaChunk + B + 1;
  return chunks * H * d * dv + (per_channel ? chunks * H * d + (long)rows * H * d + 8 : 0) + 8;
}

// Returns 1 (nothing launched) for sizes it does not take, 2 when the workspace is too small.
extern "C" int dlia_linear_attention(void* out, int out_f32, long ldo, const float* z, long ldz, float* state, const float* head_decay,
                                     const float* a2t, const float* a_b, int rank, const float* norm_w, const int* q_start, const int* ctx,
                                     const int* slots, int B, int T, int max_q, int H, int d, int dv, int state_rows, int col_q, int col_k,
                                     int col_v, int col_g, int col_a, float qscale, float inv_tau, float eps, float* ws, long ws_floats,
                                     hipStream_t stream) {
  if (B <= 0 || max_q <= 0 || T <= 0) return 0;
  if (d < 1 || dv < 1 || d > 512 || dv > 512) return 1;
  LaArgs p;
  p.out = out; p.ldo = ldo; p.z = z; p.ldz = ldz; p.state = state; p.head_decay = head_decay; p.a2t = a2t; p.a_b = a_b; p.norm_w = norm_w;
  p.q_start = q_start; p.ctx = ctx; p.slots = slots; p.H = H; p.d = d; p.dv = dv; p.rank = rank; p.state_rows = state_rows;
  p.col_q = col_q; p.col_k = col_k; p.col_v = col_v; p.col_g = col_g; p.col_a = col_a; p.qscale = qscale; p.inv_tau = inv_tau; p.eps = eps;
  p.nblk = (d + kLaCh - 1) / kLaCh;
  p.ws_state = p.ws_dec = p.g = nullptr;
  const bool vec = dv % 4 == 0 && (uintptr_t)state % 16 == 0;
  p.vec = dv % 4 == 0 && col_v % 4 == 0 && ldz % 4 == 0 && (uintptr_t)z % 16 == 0;
  if (max_q == 1) {
    const bool v4 = vec && p.vec;
    const int units = v4 ? dv / 4 : dv, CT = units < 256 ? units : 256;
    const size_t lds = ((3 * d + 3) / 4 * 4 + (256 / CT) * dv) * sizeof(float);
    const dim3 grid(H, B);
    if (out_f32) {
      if (v4) hipLaunchKernelGGL((la_decode_kernel<float, 4>), grid, dim3(256), lds, stream, p);
      else hipLaunchKernelGGL((la_decode_kernel<float, 1>), grid, dim3(256), lds, stream, p);
    } else {
      if (v4) hipLaunchKernelGGL((la_decode_kernel<bf16, 4>), grid, dim3(256), lds, stream, p);
      else hipLaunchKernelGGL((la_decode_kernel<bf16, 1>), grid, dim3(256), lds, stream, p);
    }
    return 0;
  }
  if (!ws || ws_floats < dlia_linear_attention_ws_floats(T, B, H, d, dv, head_decay ? 0 : 1)) return 2;
  const long chunks = (long)T / kLaChunk + B + 1;
  p.ws_state = ws;
  if (!head_decay) { p.ws_dec = ws + (chunks * H * d * dv + 3) / 4 * 4; p.g = p.ws_dec + (chunks * H * d + 3) / 4 * 4; }
  const int nc = (max_q + kLaChunk - 1) / kLaChunk;
  hipLaunchKernelGGL(la_local_kernel, dim3(H, B, nc * p.nblk), dim3(256), 0, stream, p);
  const long size = (long)d * dv;
  if (vec && (uintptr_t)ws % 16 == 0) hipLaunchKernelGGL((la_carry_kernel<4>), dim3((size + 1023) / 1024, H, B), dim3(256), 0, stream, p);
  else hipLaunchKernelGGL((la_carry_kernel<1>), dim3((size + 255) / 256, H, B), dim3(256), 0, stream, p);
  const dim3 grid(H, B, nc);
#define DLIA_LA(OT, NCT)                                                                                          \
  do {                                                                                                            \
    if (head_decay) hipLaunchKernelGGL((la_out_kernel<OT, NCT, true>), grid, dim3(512), 0, stream, p);            \
    else hipLaunchKernelGGL((la_out_kernel<OT, NCT, false>), grid, dim3(512), 0, stream, p);                      \
  } while (0)
  if (out_f32) { if (dv <= 128) DLIA_LA(float, 1); else if (dv <= 256) DLIA_LA(float, 2); else DLIA_LA(float, 4); }
  else { if (dv <= 128) DLIA_LA(bf16, 1); else if (dv <= 256) DLIA_LA(bf16, 2); else DLIA_LA(bf16, 4); }
#undef DLIA_LA
  return 0;
}
