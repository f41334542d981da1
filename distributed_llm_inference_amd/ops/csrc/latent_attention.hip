// Attention of many query heads over ONE cached row per token (a latent followed by a rotated key part; the values are the
// latent, i.e. the row's first entries), on the matrix cores, bf16, with an optional sliding window.
//
// Queries carry the key up-projection (H rows of D entries per token, a token's rows side by side), so the heads of a token are
// just more query rows over the same keys: a sequence's n tokens are n H consecutive rows, row r belongs to token r / H, and a
// workgroup takes consecutive rows whatever the head count.
//   prompt steps   eight waves (four for the longest rows) of 16 rows each; a row's output lies in its wave's registers (DVT accumulator tiles)
//   SPLITV         (steps of single tokens, 16 rows per workgroup) all four waves form the same 16 rows' scores and each owns a
//                  quarter of the value entries: few rows over many bytes, so the waves share the loads, not the arithmetic
// Both walk the cache block by block (32 tokens): the block's key rows (contiguous in the cache) and its key-contiguous value
// copy are brought into one half of an LDS double buffer by direct loads (no register round trip) while the other half is
// multiplied; one barrier per block.
//   Key rows: rows of NC 16-byte pieces; piece c of row r sits at place c ^ f(r), f(r) = r % 4 + 4 (r / 8 % 2), so that the 16 rows
//   a fragment reads at one piece spread over all banks. The direct loads land linearly, so the places are permuted on the
//   address side. Score tile tl takes the keys 8 (m / 4) + m % 4 + 4 tl as its rows m: a lane then holds the scores of EIGHT
//   CONSECUTIVE keys of one query, which as weights are the B fragment of the value product whose A fragment is 16 contiguous
//   bytes of a value row.
// The running maximum only moves when a score exceeds it by 8 (in units of log2): weights stay below 2^8 and the accumulators
// are rescaled a few times per row instead of once per block. The key blocks of a workgroup's rows can be dealt out to
// gridDim.y workgroups, each leaving (maximum, sum, weighted values) per row for tile_merge.
#include "common.h"
#include "launch.h"

namespace dlia {

constexpr int kLatBlock = 32;          // tokens per cache block
constexpr float kLatLn2 = 0.6931471805599453f, kLatLog2e = 1.4426950408889634f;

struct LatArgs {
  bf16* out; const bf16* q; const bf16* kcache; const bf16* vt; float* part;
  const int* q_start; const int* ctx; const int* slots; const int* block_table;
  int tiles_per_seq, max_blocks, num_blocks, table_rows, H, D, R, window;
  float scale;
};

// bytes of one half of the double buffer
template <int KS, int DVT> constexpr int lat_bytes() { return KS * 2048 + DVT * 1024; }
// waves of a workgroup: eight, or four where 16 rows' queries and accumulators want more than half of the register file
template <int KS, bool SPLITV> constexpr int lat_waves() { return SPLITV || KS > 16 ? 4 : 8; }

template <int KS, int DVT, bool SPLITV>
__global__ __launch_bounds__((64 * lat_waves<KS, SPLITV>())) void latent_attention_kernel(LatArgs p) {
  extern __shared__ __attribute__((aligned(1024))) char smem[];
  constexpr int NC = KS * 4, KP = KS * 2, RUNS = (KP + DVT) / 4, NW = lat_waves<KS, SPLITV>(), MYRUNS = (RUNS + NW - 1) / NW, BUF = lat_bytes<KS, DVT>();
  constexpr int CT = SPLITV ? DVT / 4 : DVT;                 // accumulator tiles of a wave
  static_assert(KP % 4 == 0 && DVT % 4 == 0 && NC % 8 == 0, "whole runs of four pieces");
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r16 = lane & 15, kq = lane >> 4;
  const int b = blockIdx.x / p.tiles_per_seq, ti = blockIdx.x % p.tiles_per_seq;
  const int t0 = p.q_start[b], n = p.q_start[b + 1] - t0, c0 = p.ctx[b], slot = p.slots[b];
  const int H = p.H, D = p.D, R = p.R, rows = n * H;
  const int w0 = ti * (SPLITV ? 16 : 16 * NW);               // first row of the workgroup
  if (w0 >= rows || n <= 0 || slot < 0 || slot >= p.table_rows) return;      // (whole workgroup)
  const int w1 = min(rows, w0 + (SPLITV ? 16 : 16 * NW));
  const int r0 = SPLITV ? w0 : w0 + wave * 16;          // first row of the wave
  const int pos_first = c0 + w0 / H, pos_last = c0 + (w1 - 1) / H;
  const long row0 = (long)t0 * H;                            // the sequence's first row in q and out
  // queries: B fragments of the whole kernel
  u32x4 qf[KS];
  int qpos; bool qok;
  {
    const int r = r0 + r16;
    qok = r < w1;
    qpos = c0 + (qok ? r : w0) / H;
    const bf16* qr = p.q + (row0 + (qok ? r : w0)) * D;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int c = k * 32 + kq * 8;
      qf[k] = qok && c < D ? ld16(qr + c) : u32x4{0u, 0u, 0u, 0u};
    }
  }
  float m = -INFINITY, ls = 0.f;
  f32x4 o[CT];
#pragma unroll
  for (int c = 0; c < CT; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  // byte offsets (from the block's key rows / value rows) of the pieces this lane brings: runs wave, wave + NW, ... of four pieces
  const int nc = D / 8;
  unsigned off[MYRUNS][4];
#pragma unroll
  for (int i = 0; i < MYRUNS; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int piece = (wave + NW * i) * 4 + j;
      if (piece < KP) {
        const int L = piece * 64 + lane, row = L / NC, cs = L % NC;
        int c = cs ^ ((row & 3) | ((row >> 1) & 4));
        if (c >= nc) c = 0;                                  // (places beyond the row: finite entries that meet zero query entries)
        off[i][j] = (unsigned)(row * D * 2 + c * 16);
      } else {
        const int L = (piece - KP) * 64 + lane, row = L >> 2;
        off[i][j] = (unsigned)((row < R ? row : 0) * (kLatBlock * 2) + (L & 3) * 16);
      }
    }
  const int* table = p.block_table + (long)slot * p.max_blocks;
  const unsigned lds0 = (unsigned)(uintptr_t)smem;
  auto bring = [&](int blk, int half) {
    const char* kb = reinterpret_cast<const char*>(p.kcache + (long)blk * kLatBlock * D);
    const char* vb = reinterpret_cast<const char*>(p.vt + (long)blk * R * kLatBlock);
#pragma unroll
    for (int i = 0; i < MYRUNS; ++i) {
      const int run = wave + NW * i;
      if (run < RUNS) {
        const char* base = run * 4 < KP ? kb : vb;
        const void* g[4] = {base + off[i][0], base + off[i][1], base + off[i][2], base + off[i][3]};
        lds_dma_run<4>(g, lds0 + half * BUF + run * 4096);
      }
    }
  };
  const int lo = p.window > 0 ? max(0, pos_first - p.window + 1) : 0;
  const int kb_hi = min(pos_last / kLatBlock, p.max_blocks - 1), step = gridDim.y;
  auto block_at = [&](int kb) { return __builtin_amdgcn_readfirstlane(table[min(kb, kb_hi)]); };     // the cache block of the kb-th 32 tokens
  auto valid = [&](int blk) { return blk >= 0 && blk < p.num_blocks; };        // (a block that is not there: any block's rows, all masked)
  auto fetch = [&](int blk, int h2) { bring(valid(blk) ? blk : 0, h2); };
  const float sl2 = p.scale * kLatLog2e;
  int kb = lo / kLatBlock + blockIdx.y, half = 0;
  if (kb > kb_hi) kb = kb_hi + 1;
  int cur = block_at(kb);
  if (kb <= kb_hi) fetch(cur, 0);
  for (; kb <= kb_hi; kb += step) {
    const int nxt = block_at(kb + step);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                                         // this half has arrived for all waves, the other one is consumed
    if (kb + step <= kb_hi) fetch(nxt, half ^ 1);
    const char* kl = smem + half * BUF;
    const char* vl = kl + KS * 2048;
    f32x4 s[2];
    s[0] = s[1] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int krow = (r16 >> 2) * 8 + (r16 & 3);
    // fragments of KG k-steps on their way while those of the group before are multiplied (the scheduler is kept from
    // hoisting all of them, which the registers do not hold beside the accumulators)
    constexpr int KG = KS == 16 && !SPLITV ? 2 : KS % 4 == 0 ? 4 : 3, VG = CT % 4 == 0 ? 4 : CT % 7 == 0 ? 7 : CT % 3 == 0 ? 3 : 2;
    static_assert(KS % KG == 0 && CT % VG == 0, "whole groups");
    u32x4 kf[2][KG][2], vf[2][VG];
    auto load_k = [&](int g) {
#pragma unroll
      for (int u = 0; u < KG; ++u) {
        const int c = (((g * KG + u) * 4 + kq) ^ (r16 & 7)) * 16;
        kf[g & 1][u][0] = *reinterpret_cast<const u32x4*>(kl + krow * (NC * 16) + c);
        kf[g & 1][u][1] = *reinterpret_cast<const u32x4*>(kl + (krow + 4) * (NC * 16) + c);
      }
    };
    auto load_v = [&](int g) {
#pragma unroll
      for (int u = 0; u < VG; ++u) {
        const int tile = (SPLITV ? wave * CT : 0) + g * VG + u;
        vf[g & 1][u] = *reinterpret_cast<const u32x4*>(vl + (tile * 16 + r16) * 64 + kq * 16);
      }
    };
    load_k(0);
#pragma unroll
    for (int g = 0; g < KS / KG; ++g) {
      if (g + 1 < KS / KG) load_k(g + 1);
      else load_v(0);
#pragma unroll
      for (int u = 0; u < KG; ++u) {
        s[0] = mfma16(kf[g & 1][u][0], qf[g * KG + u], s[0]);
        s[1] = mfma16(kf[g & 1][u][1], qf[g * KG + u], s[1]);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    const int j0 = kb * kLatBlock;
    const bool there = valid(cur);
    const int far = p.window > 0 ? p.window : 0x7fffffff;
    u32x4 pf;
    {
      float x[8], bm = -INFINITY;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int back = qpos - (j0 + kq * 8 + i);      // visible: 0 <= back < window
        x[i] = there && back >= 0 && back < far ? s[i >> 2][i & 3] * sl2 : -INFINITY;
        bm = fmaxf(bm, x[i]);
      }
      bm = fmaxf(bm, __shfl_xor(bm, 16, 64));
      bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
      if (__any(bm > m + 8.f)) {
        const float mn = fmaxf(m, bm), corr = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - mn);
        ls *= corr;
#pragma unroll
        for (int c = 0; c < CT; ++c) o[c] *= corr;
        m = mn;
      }
      const float mm = m == -INFINITY ? 0.f : m;
      float add = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) { x[i] = __builtin_amdgcn_exp2f(x[i] - mm); add += x[i]; }
      ls += add;
      pf = pack8(x);
    }
#pragma unroll
    for (int g = 0; g < CT / VG; ++g) {
      if (g + 1 < CT / VG) load_v(g + 1);
#pragma unroll
      for (int u = 0; u < VG; ++u) o[g * VG + u] = mfma16(vf[g & 1][u], pf, o[g * VG + u]);
      __builtin_amdgcn_sched_barrier(0);
    }
    cur = nxt;
    half ^= 1;
  }
  ls += __shfl_xor(ls, 16, 64);
  ls += __shfl_xor(ls, 32, 64);
  if (!qok) return;
  const long row = row0 + r0 + r16;
  if (p.part) {
    float* pr = p.part + (row * step + blockIdx.y) * (R + 2);
    if (kq == 0 && (!SPLITV || wave == 0)) { pr[R] = m == -INFINITY ? m : m * kLatLn2; pr[R + 1] = ls; }
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int col = (SPLITV ? wave * CT + c : c) * 16 + kq * 4;
      if (col >= R) break;
#pragma unroll
      for (int r = 0; r < 4; ++r) pr[col + r] = o[c][r];
    }
    return;
  }
  const float inv = ls > 0.f ? 1.f / ls : 0.f;
  bf16* orow = p.out + row * R;
#pragma unroll
  for (int c = 0; c < CT; ++c) {
    const int col = (SPLITV ? wave * CT + c : c) * 16 + kq * 4;
    if (col >= R) break;
    *reinterpret_cast<u32x2*>(orow + col) = u32x2{pack_bf16(o[c][0] * inv, o[c][1] * inv), pack_bf16(o[c][2] * inv, o[c][3] * inv)};
  }
}

template <int KS, int DVT>
static int launch_latent(const LatArgs& p, bool single, dim3 grid, hipStream_t stream) {
  const int lds = 2 * lat_bytes<KS, DVT>();
  if (single) {
    static const hipError_t ok = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attention_kernel<KS, DVT, true>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (ok != hipSuccess) return 1;
    hipLaunchKernelGGL((latent_attention_kernel<KS, DVT, true>), grid, dim3(256), lds, stream, p);
  } else {
    static const hipError_t ok = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attention_kernel<KS, DVT, false>),
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (ok != hipSuccess) return 1;
    hipLaunchKernelGGL((latent_attention_kernel<KS, DVT, false>), grid, dim3((64 * lat_waves<KS, false>())), lds, stream, p);
  }
  return 0;
}

}  // namespace dlia

using namespace dlia;

// Sizes in whole 16-byte pieces, rows up to 576 entries of which up to 512 are values.
extern "C" int dlia_latent_attention_fits(int D, int R) { return D % 8 == 0 && R % 8 == 0 && R >= 8 && R <= D && D <= 576 && R <= 512; }

static int latent_variant(int D, int R) {
  if (D <= 128 && R <= 128) return 0;
  if (D <= 256 && R <= 256) return 1;
  if (D <= 384 && R <= 384) return 2;
  if (D <= 512 && R <= 448) return 3;
  return 4;
}

// Workgroups a tile's key blocks are dealt out to: enough for the chip when a step has few rows.
static int latent_splits(long groups) {
  int z = 1;
  while (z < 16 && groups * z * 2 <= 256) z <<= 1;
  return z;
}
static long latent_tiles(int D, int R, int max_q, int H) {
  const int per = max_q == 1 ? 16 : latent_variant(D, R) == 4 ? 64 : 128;
  return ((long)max_q * H + per - 1) / per;
}

// Floats of the workspace with which any step of up to `rows` tokens in up to B sequences may use its splits.
extern "C" long dlia_latent_attention_part_floats(int rows, int B, int H, int R) {
  const long most = (long)rows * H, cap = 256L * 128 + 16L * 128;      // (splits are used while their workgroups are at most 256)
  return (most * 16 < cap ? most * 16 : cap) * (R + 2);
}

// q [T][H][D] and out [T][H][R] contiguous, keys [blocks][32][D], values [blocks][R][32]. Returns 1 (nothing launched) for sizes it
// does not take.
extern "C" int dlia_latent_attention(void* out, const void* q, const void* kcache, const void* vt, const int* q_start, const int* ctx,
                                     const int* slots, const int* block_table, int B, int T, int max_q, int max_blocks, int num_blocks,
                                     int table_rows, int H, int D, int R, float scale, int window, float* part, long part_floats,
                                     hipStream_t stream) {
  if (B <= 0 || max_q <= 0 || T <= 0) return 0;
  if (!dlia_latent_attention_fits(D, R)) return 1;
  LatArgs p;
  p.out = (bf16*)out; p.q = (const bf16*)q; p.kcache = (const bf16*)kcache; p.vt = (const bf16*)vt; p.part = nullptr;
  p.q_start = q_start; p.ctx = ctx; p.slots = slots; p.block_table = block_table;
  const long tiles = latent_tiles(D, R, max_q, H);
  p.tiles_per_seq = (int)tiles; p.max_blocks = max_blocks; p.num_blocks = num_blocks; p.table_rows = table_rows;
  p.H = H; p.D = D; p.R = R; p.window = window; p.scale = scale;
  int nz = latent_splits(B * tiles);
  while (nz > 1 && (!part || part_floats < (long)T * H * nz * (R + 2))) nz >>= 1;
  if (nz > 1) p.part = part;
  const dim3 grid((unsigned)(B * tiles), nz);
  const bool single = max_q == 1;
  int rc = 1;
  switch (latent_variant(D, R)) {
    case 0: rc = launch_latent<4, 8>(p, single, grid, stream); break;
    case 1: rc = launch_latent<8, 16>(p, single, grid, stream); break;
    case 2: rc = launch_latent<12, 24>(p, single, grid, stream); break;
    case 3: rc = launch_latent<16, 28>(p, single, grid, stream); break;
    default: rc = launch_latent<18, 32>(p, single, grid, stream); break;
  }
  if (rc) return rc;
  if (nz > 1) dlia_tile_merge(out, (long)H * R, part, T * H, H, R, nz, nullptr, 0, nullptr, stream);
  return 0;
}
