// Row kernels of stacks with plain-weight RMS norms before and after every sublayer of an fp32 residual stream,
//     x <- x + m rms(f(rms(x) w)) wb,
// whose embedding adds a row chosen by (previous token, token), whose repeated stretch of layers starts every pass from a linear
// map of the stream beside the embedding output, and whose attention mixers norm every head's query and key.
//
//   embed_bigram   x0 = table[token] * scale + bigram[hash(previous token, token)] in fp32, and in the GEMMs' type as one half of
//                  the rows the pass map reads. The previous token of a portion's first token comes from the sequence's cache
//                  blocks: every token's id is written to its place in a page of 32 ids per block, the way keys and values are,
//                  so it needs no slot state, moves with the block table, and a step that is run twice writes the same.
//   sandwich_join  one launch per sublayer boundary: the finished sublayer's output (a GEMM's, whole or as the partial sums of its
//                  key splits, plus the token's routed expert rows) is RMS-normed over the row, weighted (the residual multiplier rides in the
//                  weight) and added to the stream; the next sublayer's normed input leaves in the GEMMs' type, or the stream
//                  itself does (the other half of the pass map's rows). A row stays in registers from its load to its store.
//   qk_prep        between an attention mixer's input projection and its cache: per head RMS norm of q and k with a weight ahead of
//                  the rotation and / or without one behind it, rotation of the first `dims` entries (pairs (2i, 2i + 1) or
//                  (i, i + dims / 2), angles from a table by position), values from columns of their own or the keys as
//                  projected. q leaves for the attention kernel, k and v go to the paged cache in the layout that kernel reads.
//                  A head's vector lies in 8 to 64 neighbouring lanes; partners of the rotation meet in LDS.
//   relu_act       relu(z)^2, or relu(gate) * up from gate | up side by side
// Statistics, rotation and the stream are fp32; outputs take the GEMMs' / the cache's type (bf16 or fp32).
#include "units.h"
#include "kv_layout.h"
#include "launch.h"

namespace dlia {

constexpr int kSandThreads = 256;

// ---- embedding -------------------------------------------------------------------------------------------------------
template <typename TT>
__global__ __launch_bounds__(kSandThreads) void embed_bigram_kernel(
    float* __restrict__ out, TT* __restrict__ cat, long ldc, int cat_both, const int* __restrict__ ids, const TT* __restrict__ table,
    float scale, const TT* __restrict__ bigram, int buckets, long mul_prev, long mul_cur, int* __restrict__ pages,
    const int* __restrict__ tok_pos, const int* __restrict__ tok_seq, const int* __restrict__ block_table, int max_blocks, int num_blocks,
    int table_rows, int H, int vocab) {
  const int t = blockIdx.x;
  auto clamped = [&](int v) { return v < 0 ? 0 : (v >= vocab ? vocab - 1 : v); };    // never fault on a bad id
  const int id = clamped(ids[t]);
  const TT* src = table + (long)id * H;
  const TT* bsrc = nullptr;
  if (bigram) {
    const int pos = tok_pos[t], slot = tok_seq[t];
    auto block_of = [&](int p) {
      int b = -1;
      if (slot >= 0 && slot < table_rows && p >= 0 && p / kBlockTokens < max_blocks) b = block_table[(long)slot * max_blocks + p / kBlockTokens];
      return b < num_blocks ? b : -1;
    };
    long row = buckets;                     // a sequence's first token
    if (pos > 0) {
      int prev = 0;
      if (t > 0 && tok_seq[t - 1] == slot && tok_pos[t - 1] == pos - 1) prev = ids[t - 1];
      else {
        const int b = block_of(pos - 1);
        if (b >= 0) prev = pages[(long)b * kBlockTokens + (pos - 1) % kBlockTokens];
      }
      row = ((long)clamped(prev) * mul_prev + (long)id * mul_cur) % buckets;
    }
    bsrc = bigram + row * H;
    if (threadIdx.x == 0) {
      const int b = block_of(pos);
      if (b >= 0) pages[(long)b * kBlockTokens + pos % kBlockTokens] = id;
    }
  }
  float* dst = out + (long)t * H;
  for (int i = threadIdx.x; i < H; i += kSandThreads) {
    float v = (float)src[i] * scale;
    if (bsrc) v += (float)bsrc[i];
    dst[i] = v;
    if (cat) {
      cat[(long)t * ldc + H + i] = (TT)v;
      if (cat_both) cat[(long)t * ldc + i] = (TT)v;
    }
  }
}

// ---- sublayer boundary -----------------------------------------------------------------------------------------------
template <typename OT, int V, int NR>
__global__ __launch_bounds__(kSandThreads) void sandwich_join_kernel(
    OT* __restrict__ out, long ldo, float* __restrict__ x, long ldx, const float* __restrict__ ya, long ldya, int ya_parts, long ya_step,
    const float* __restrict__ ey, const int* __restrict__ pair_row, int top, const float* __restrict__ wb,
    const float* __restrict__ wn, int H, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, units = H / V, nt = blockDim.x;
  float* xr = x + (long)t * ldx;
  Unit<V> xv[NR];
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int u = threadIdx.x + k * nt;
    if (u < units) xv[k] = ldu<V>(xr + u * V);
  }
  if (wb) {
    Unit<V> y[NR];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NR; ++k) {
      const int u = threadIdx.x + k * nt;
      if (u >= units) break;
      const int c = u * V;
#pragma unroll
      for (int e = 0; e < V; ++e) y[k].v[e] = 0.f;
      if (ya) {
        const float* yr = ya + (long)t * ldya + c;
#pragma unroll 4
        for (int i = 0; i < ya_parts; ++i) {
          const Unit<V> a = ldu<V>(yr + i * ya_step);
#pragma unroll
          for (int e = 0; e < V; ++e) y[k].v[e] += a.v[e];
        }
      }
      if (ey)
        for (int i = 0; i < top; ++i) {
          const int er = pair_row[(long)t * top + i];
          if (er < 0) continue;
          const Unit<V> a = ldu<V>(ey + (long)er * H + c);
#pragma unroll
          for (int e = 0; e < V; ++e) y[k].v[e] += a.v[e];
        }
#pragma unroll
      for (int e = 0; e < V; ++e) ss += y[k].v[e] * y[k].v[e];
    }
    ss = block_sum(ss, scratch);
    const float r = 1.f / sqrtf(ss / H + eps);
#pragma unroll
    for (int k = 0; k < NR; ++k) {
      const int u = threadIdx.x + k * nt;
      if (u >= units) break;
      const Unit<V> w = ldu<V>(wb + u * V);
#pragma unroll
      for (int e = 0; e < V; ++e) xv[k].v[e] += y[k].v[e] * r * w.v[e];
      stu<V>(xr + u * V, xv[k]);
    }
  }
  if (!out) return;
  OT* orow = out + (long)t * ldo;
  float f = 1.f;
  if (wn) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NR; ++k) {
      if ((int)threadIdx.x + k * nt >= units) break;
#pragma unroll
      for (int e = 0; e < V; ++e) ss += xv[k].v[e] * xv[k].v[e];
    }
    ss = block_sum(ss, scratch);
    f = 1.f / sqrtf(ss / H + eps);
  }
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int u = threadIdx.x + k * nt;
    if (u >= units) break;
    Unit<V> o = xv[k];
    if (wn) {
      const Unit<V> w = ldu<V>(wn + u * V);
#pragma unroll
      for (int e = 0; e < V; ++e) o.v[e] *= f * w.v[e];
    }
    stu<V>(orow + u * V, o);
  }
}

// ---- queries, keys and values of an attention mixer --------------------------------------------------------------------
struct PrepParams {
  const void* z; long ldz;              // [T, q | k (| v) ...]
  int T, H, G, d, dv, col_v;            // col_v < 0: the values are the keys as projected
  const float *qw, *kw; int unit; float eps;
  int dims, interleaved; const float *cos_t, *sin_t; int table_pos;
  int whole;                            // rotated parts come in whole runs of V entries: vector reads of partners and angles
  void* q_out; long ldqo;
  void* kc; void* vc; int layout;       // 0: rows of k and of v; 1: values key-contiguous; 2: the fragment-ordered slabs (kv_layout.h)
  const int *tok_pos, *tok_seq, *block_table; int max_blocks, num_blocks, table_rows;
};

template <typename T, int V>
__device__ __forceinline__ void load_vals(const T* p, float (&f)[V]) {
  if constexpr (V == 8 && sizeof(T) == 2) {
    unpack8(ld16(p), f);
  } else if constexpr (V == 8) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) { f[j] = a[j]; f[4 + j] = b[j]; }
  } else {
    f[0] = (float)p[0];
  }
}
template <typename T, int V>
__device__ __forceinline__ void store_vals(T* p, const float (&f)[V]) {
  if constexpr (V == 8 && sizeof(T) == 2) {
    st16(p, pack8(f));
  } else if constexpr (V == 8) {
    *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{f[4], f[5], f[6], f[7]};
  } else {
    p[0] = (T)f[0];
  }
}

template <int LPH>
__device__ __forceinline__ float lanes_sum(float v) {
#pragma unroll
  for (int o = LPH / 2; o >= 1; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// LPH lanes per head vector, V consecutive entries per lane and chunk, NCH chunks.
template <typename ZT, typename QT, typename CT, int V, int LPH, int NCH>
__global__ __launch_bounds__(kSandThreads) void qk_prep_kernel(PrepParams p) {
  extern __shared__ __attribute__((aligned(16))) float rows[];
  constexpr int GPB = kSandThreads / LPH;
  const int grp = threadIdx.x / LPH, l = threadIdx.x % LPH;
  const int per_tok = p.H + p.G + (p.col_v >= 0 ? p.G : 0);
  const long item = (long)blockIdx.x * GPB + grp;
  const bool live = item < (long)p.T * per_tok;
  const long t = live ? item / per_tok : 0;
  const int hv = live ? (int)(item % per_tok) : 0;
  const bool is_q = hv < p.H, is_v = hv >= p.H + p.G;
  const int head = is_q ? hv : is_v ? hv - p.H - p.G : hv - p.H;
  const int n = is_v ? p.dv : p.d;                                // entries of this vector
  const int col = is_v ? p.col_v + head * p.dv : hv * p.d;
  const int pos = p.tok_pos[t], slot = p.tok_seq[t];
  const ZT* src = reinterpret_cast<const ZT*>(p.z) + t * p.ldz + col;
  float f[NCH][V];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (c * LPH + l) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) f[c][e] = 0.f;
    if (live && i < n) load_vals<ZT, V>(src + i, f[c]);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += f[c][e] * f[c][e];
  }
  // where the token's cache rows lie (an unallocated place is skipped, never a wild store)
  int blk = -1;
  if (live && !is_q && slot >= 0 && slot < p.table_rows && pos >= 0 && pos / kBlockTokens < p.max_blocks)
    blk = p.block_table[(long)slot * p.max_blocks + pos / kBlockTokens];
  const bool store = blk >= 0 && blk < p.num_blocks;
  const int off = store ? pos % kBlockTokens : 0;
  if (store && (is_v || p.col_v < 0)) {          // values: as projected
    CT* vb = reinterpret_cast<CT*>(p.layout == 2 ? p.kc : p.vc);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * LPH + l) * V;
      if (i >= p.dv) break;
      if (p.layout == 0) {
        store_vals<CT, V>(vb + (((long)blk * p.G + head) * kBlockTokens + off) * p.dv + i, f[c]);
      } else if (p.layout == 1) {
#pragma unroll
        for (int e = 0; e < V; ++e) vb[(((long)blk * p.G + head) * p.dv + i + e) * kBlockTokens + off] = (CT)f[c][e];
      } else {
        CT* base = vb + kv_head_base(blk, head, p.G, p.d, 1);
#pragma unroll
        for (int e = 0; e < V; ++e) base[v_elem_off(off, i + e)] = (CT)f[c][e];
      }
    }
  }
  const float* w = is_q ? p.qw : p.kw;
  if (p.qw && !is_v) {
    ss = lanes_sum<LPH>(ss);
    const float r = 1.f / sqrtf(ss / n + p.eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * LPH + l) * V;
#pragma unroll
      for (int e = 0; e < V; ++e)
        if (i + e < n) f[c][e] *= r * w[i + e];
    }
  }
  if (p.dims > 0) {
    float* row = rows + grp * ((p.d + 3) / 4 * 4 + 4);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * LPH + l) * V;
      if (!is_v && i < p.d && !(p.whole && p.interleaved)) store_vals<float, V>(row + i, f[c]);
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    if (!is_v && live && pos >= 0 && pos < p.table_pos) {
      const int half = p.dims >> 1;
      const float* cs = p.cos_t + (long)pos * half;
      const float* sn = p.sin_t + (long)pos * half;
#pragma unroll
      for (int c = 0; c < NCH; ++c) {
        const int i0 = (c * LPH + l) * V;
        if constexpr (V == 8) {
          if (p.whole) {
            if (i0 >= p.dims) break;
            if (p.interleaved) {                    // four pairs of this lane's own
              const f32x4 cv = *reinterpret_cast<const f32x4*>(cs + (i0 >> 1)), sv = *reinterpret_cast<const f32x4*>(sn + (i0 >> 1));
#pragma unroll
              for (int e = 0; e < 4; ++e) {
                const float u = f[c][2 * e], v = f[c][2 * e + 1];
                f[c][2 * e] = u * cv[e] - v * sv[e];
                f[c][2 * e + 1] = v * cv[e] + u * sv[e];
              }
            } else {                                // eight entries against the partner run of the other half
              const bool first = i0 < half;
              const int pi = first ? i0 : i0 - half;
              float o[8], cv[8], sv[8];
              load_vals<float, 8>(row + (first ? i0 + half : pi), o);
              load_vals<float, 8>(cs + pi, cv);
              load_vals<float, 8>(sn + pi, sv);
#pragma unroll
              for (int e = 0; e < 8; ++e) f[c][e] = f[c][e] * cv[e] + (first ? -o[e] : o[e]) * sv[e];
            }
            continue;
          }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) {
          const int i = i0 + e;
          if (i < p.dims) {
            const bool first = p.interleaved ? !(i & 1) : i < half;
            const int pi = p.interleaved ? i >> 1 : (first ? i : i - half);
            const float other = row[p.interleaved ? i ^ 1 : (first ? i + half : i - half)];
            f[c][e] = f[c][e] * cs[pi] + (first ? -other : other) * sn[pi];
          }
        }
      }
    }
  }
  if (p.unit && !is_v) {
    float s2 = 0.f;
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < V; ++e) s2 += f[c][e] * f[c][e];
    s2 = lanes_sum<LPH>(s2);
    const float r = 1.f / sqrtf(s2 / p.d + p.eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < V; ++e) f[c][e] *= r;
  }
  if (!live || is_v) return;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (c * LPH + l) * V;
    if (i >= p.d) break;
    if (is_q) {
      store_vals<QT, V>(reinterpret_cast<QT*>(p.q_out) + t * p.ldqo + (long)head * p.d + i, f[c]);
    } else if (store) {
      CT* kb = reinterpret_cast<CT*>(p.kc);
      if (p.layout == 2) store_vals<CT, V>(kb + kv_head_base(blk, head, p.G, p.d, 0) + k_elem_off(off, i, p.d), f[c]);
      else store_vals<CT, V>(kb + (((long)blk * p.G + head) * kBlockTokens + off) * p.d + i, f[c]);
    }
  }
}

// ---- activation ------------------------------------------------------------------------------------------------------
template <typename ZT, typename OT, int V>
__global__ __launch_bounds__(256) void relu_act_kernel(OT* __restrict__ act, long lda, const ZT* __restrict__ z, long ldz, int F, int glu) {
  const long m = blockIdx.y;
  const int c = (blockIdx.x * 256 + threadIdx.x) * V;
  if (c >= F) return;
  float a[V], u[V];
  load_vals<ZT, V>(z + m * ldz + c, a);
  if (glu) load_vals<ZT, V>(z + m * ldz + F + c, u);
#pragma unroll
  for (int e = 0; e < V; ++e) { const float r = fmaxf(a[e], 0.f); a[e] = r * (glu ? u[e] : r); }
  store_vals<OT, V>(act + m * lda + c, a);
}

}  // namespace dlia

using namespace dlia;

extern "C" void dlia_embed_bigram(float* out, void* cat, long ldc, int cat_both, const int* ids, const void* table, int f32, float scale,
                                  const void* bigram, int buckets, long mul_prev, long mul_cur, int* pages, const int* tok_pos,
                                  const int* tok_seq, const int* block_table, int T, int max_blocks, int num_blocks, int table_rows, int H,
                                  int vocab, hipStream_t stream) {
  if (T <= 0) return;
  if (f32)
    hipLaunchKernelGGL(embed_bigram_kernel<float>, dim3(T), dim3(kSandThreads), 0, stream, out, (float*)cat, ldc, cat_both, ids,
                       (const float*)table, scale, (const float*)bigram, buckets, mul_prev, mul_cur, pages, tok_pos, tok_seq, block_table,
                       max_blocks, num_blocks, table_rows, H, vocab);
  else
    hipLaunchKernelGGL(embed_bigram_kernel<bf16>, dim3(T), dim3(kSandThreads), 0, stream, out, (bf16*)cat, ldc, cat_both, ids,
                       (const bf16*)table, scale, (const bf16*)bigram, buckets, mul_prev, mul_cur, pages, tok_pos, tok_seq, block_table,
                       max_blocks, num_blocks, table_rows, H, vocab);
}

extern "C" int dlia_sandwich_join_max_width(int vec) { return vec ? kSandThreads * 4 * 16 : kSandThreads * 32; }

extern "C" int dlia_sandwich_join(void* out, int out_f32, long ldo, float* x, long ldx, const float* ya, long ldya, int ya_parts,
                                  long ya_step, const float* ey, const int* pair_row, int top, const float* wb, const float* wn, int T, int H,
                                  float eps, hipStream_t stream) {
  if (T <= 0) return 0;
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = H % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0 && ldya % 4 == 0 && ya_step % 4 == 0 && al(x) && al(out) && al(ya) &&
                   al(ey) && al(wb) && al(wn);
  if (H > dlia_sandwich_join_max_width(vec)) return 1;
  const int units = vec ? H / 4 : H;
  const int threads = units <= 64 ? 64 : units <= 128 ? 128 : kSandThreads;
  const int nr = (units + threads - 1) / threads;
#define DLIA_JOIN_OT(OT, V, NR)                                                                                                   \
  hipLaunchKernelGGL((sandwich_join_kernel<OT, V, NR>), dim3(T), dim3(threads), 0, stream, (OT*)out, ldo, x, ldx, ya, ldya, ya_parts, ya_step, ey, \
                     pair_row, top, wb, wn, H, eps)
#define DLIA_JOIN(V, NR)                                                                            \
  do { if (out_f32) DLIA_JOIN_OT(float, V, NR); else DLIA_JOIN_OT(bf16, V, NR); } while (0)
  if (vec) {
    if (nr <= 1) DLIA_JOIN(4, 1); else if (nr <= 2) DLIA_JOIN(4, 2); else if (nr <= 4) DLIA_JOIN(4, 4); else if (nr <= 8) DLIA_JOIN(4, 8);
    else DLIA_JOIN(4, 16);
  } else {
    if (nr <= 2) DLIA_JOIN(1, 2); else if (nr <= 8) DLIA_JOIN(1, 8); else DLIA_JOIN(1, 32);
  }
#undef DLIA_JOIN
#undef DLIA_JOIN_OT
  return 0;
}

template <typename ZT, typename QT, typename CT>
static int launch_prep(PrepParams p, hipStream_t stream) {
  auto al = [](const void* q) { return (uintptr_t)q % 16 == 0; };
  const int widest = p.d > p.dv ? p.d : p.dv;
  const long items = (long)p.T * (p.H + p.G + (p.col_v >= 0 ? p.G : 0));
  const bool vec = p.d % 8 == 0 && p.dv % 8 == 0 && p.ldz % 8 == 0 && p.ldqo % 8 == 0 && (p.col_v < 0 || p.col_v % 8 == 0) && al(p.z) &&
                   al(p.q_out) && al(p.kc) && al(p.vc);
  if (widest > 512 || (p.layout == 2 && !(vec && sizeof(CT) == 2 && p.d == p.dv && (p.d == 64 || p.d == 128)))) return 1;
  p.whole = vec && p.dims % (p.interleaved ? 8 : 16) == 0 && al(p.cos_t) && al(p.sin_t);
  const size_t row = ((p.d + 3) / 4 * 4 + 4) * sizeof(float);
#define DLIA_PREP(V, LPH, NCH)                                                                                                    \
  hipLaunchKernelGGL((qk_prep_kernel<ZT, QT, CT, V, LPH, NCH>), dim3((unsigned)((items + kSandThreads / LPH - 1) / (kSandThreads / LPH))),  \
                     dim3(kSandThreads), (kSandThreads / LPH) * row, stream, p)
  if (vec) {
    if (widest <= 64) DLIA_PREP(8, 8, 1); else if (widest <= 128) DLIA_PREP(8, 16, 1); else DLIA_PREP(8, 16, 4);
  } else {
    if (widest <= 64) DLIA_PREP(1, 64, 1); else DLIA_PREP(1, 64, 8);
  }
#undef DLIA_PREP
  return 0;
}

extern "C" int dlia_qk_prep(const void* z, int z_f32, long ldz, int T, int H, int G, int d, int dv, int col_v, const float* qw, const float* kw,
                            int unit, float eps, int dims, int interleaved, const float* cos_t, const float* sin_t, int table_pos, void* q_out,
                            int q_f32, long ldqo, void* kc, void* vc, int cache_f32, int layout, const int* tok_pos, const int* tok_seq,
                            const int* block_table, int max_blocks, int num_blocks, int table_rows, hipStream_t stream) {
  if (T <= 0) return 0;
  const PrepParams p{z, ldz, T, H, G, d, dv, col_v, qw, kw, unit, eps, dims, interleaved, cos_t, sin_t, table_pos, 0, q_out, ldqo, kc, vc, layout,
                     tok_pos, tok_seq, block_table, max_blocks, num_blocks, table_rows};
  if (cache_f32) return z_f32 && q_f32 ? launch_prep<float, float, float>(p, stream) : 1;
  if (z_f32) return q_f32 ? launch_prep<float, float, bf16>(p, stream) : launch_prep<float, bf16, bf16>(p, stream);
  return q_f32 ? 1 : launch_prep<bf16, bf16, bf16>(p, stream);
}

extern "C" void dlia_relu_act(void* act, int out_f32, long lda, const void* z, int z_f32, long ldz, int M, int F, int glu, hipStream_t stream) {
  if (M <= 0 || F <= 0) return;
  const bool vec = F % 8 == 0 && lda % 8 == 0 && ldz % 8 == 0 && (uintptr_t)act % 16 == 0 && (uintptr_t)z % 16 == 0;
  const dim3 grid((F + 256 * (vec ? 8 : 1) - 1) / (256 * (vec ? 8 : 1)), M);
#define DLIA_RELU(ZT, OT)                                                                                                            \
  do {                                                                                                                             \
    if (vec) hipLaunchKernelGGL((relu_act_kernel<ZT, OT, 8>), grid, dim3(256), 0, stream, (OT*)act, lda, (const ZT*)z, ldz, F, glu);  \
    else hipLaunchKernelGGL((relu_act_kernel<ZT, OT, 1>), grid, dim3(256), 0, stream, (OT*)act, lda, (const ZT*)z, ldz, F, glu);      \
  } while (0)
  if (out_f32) { if (z_f32) DLIA_RELU(float, float); else DLIA_RELU(bf16, float); }
  else { if (z_f32) DLIA_RELU(float, bf16); else DLIA_RELU(bf16, bf16); }
#undef DLIA_RELU
}
