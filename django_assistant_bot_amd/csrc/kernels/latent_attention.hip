// Latent attention: keys and values of every head are linear images of one cached latent per token.
//
// The paged cache holds the RMS-normed latent c only ([num_blocks, block_size, R], R = rank padded to
// 64).  Two exact forms of the same scores are used:
//   * prefill expands K = W_uk c, V = W_uv c for the chunk's visible context with one MFMA GEMM and
//     runs the flash kernel (attention.hip, windowed + sink form): 2 (dim + vdim) FLOP per score;
//   * decode absorbs W_uk into the query (q' = W_uk^T q, one small per-head GEMM) and W_uv behind the
//     softmax, so all heads attend to the SAME R-wide rows: each cached byte is read once per step and
//     serves every head (latent_decode below, HBM-bound).
// Masks: a sliding window of `window` keys (self included; 0 = unlimited).  Softmax sink: one extra
// logit per head that joins the denominator and has neither key nor value.
//
// Rotary positions (optional): a rotated part of every query head and one rotated key part shared by the heads.  The
// cached row then is [c | rotated key].  The absorbed query carries its rotated part along (an identity block in its
// weights); the expanded keys do the same, or latent_key_fill copies the part to every head.
//
//   latent_write   : split-K slabs of the [q | latent] projection -> q rows, RMS norm, rotation, cache write
//   latent_gather  : packed copy of the cached latents a prefill chunk sees (K / V expansion input)
//   latent_key_fill: the gathered rotated key part into every expanded key head
//   head_gemm      : Y[t, h, :] = W[h] X[t, h, :], weights in the ops.shuffle_weights layout
//   latent_decode  : MFMA decode over key partitions, and the combine of the partitions
//   latent_any     : one (token, head) per workgroup, any rank <= 2048, bf16 or fp32: the 32-bit mode
//                    and shapes outside the MFMA kernels' tiles
#include "common.h"
#include "launchers.h"
#include "proj.h"

namespace dab {

// ---------------------------------------------------------------------------------- latent_write

// One workgroup per token.  Wave 0: latent columns [q_cols, q_cols + R) summed over the slabs, RMS over
// the first `rank` of them, gain, cache row (slot < 0: no write).  Waves 1-3: the q columns (q_out set).
// ROPE: latent columns c_at .. c_at + rot and the columns q_at .. q_at + rot of every D-wide head are rotated, neighbours
// (2i, 2i + 1) being a pair; they take no part in the norm.  Heads and rotated parts start at multiples of 8.
template <typename YT, typename CT, bool ROPE>
__global__ __launch_bounds__(256) void latent_write_kernel(const YT* __restrict__ y, int S, long slab_stride, long ld,
                                                           CT* __restrict__ q_out, int q_cols,
                                                           const float* __restrict__ gain, CT* __restrict__ cache,
                                                           const int64_t* __restrict__ slots, int R, int rank,
                                                           float eps, LatentRope rope) {
  extern __shared__ __attribute__((aligned(16))) float2 turn[];  // (cosine, sine) of every pair, 1 / 0 past the last
  const int t = blockIdx.x, tid = threadIdx.x;
  const int rot8 = (rope.rot + 7) & ~7;
  if constexpr (ROPE) {
    const double pos = (double)rope.positions[t];
    for (int i = tid; i < rot8 / 2; i += 256) {
      float s = 0.f, c = 1.f;
      if (2 * i < rope.rot) {
        const double turns = pos * rope.freq[i];
        sincos_turn(turns - rint(turns), s, c);
        s *= rope.mul;
        c *= rope.mul;
      }
      turn[i] = make_float2(c, s);
    }
    __syncthreads();
  }
  auto rotate = [&](int d, float(&v)[8]) {  // columns d .. d + 7 of a rotated part
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float2 w = turn[d / 2 + j];
      const float a = v[2 * j], b = v[2 * j + 1];
      v[2 * j] = a * w.x - b * w.y;
      v[2 * j + 1] = b * w.x + a * w.y;
    }
  };
  const YT* row = y + (size_t)t * ld;
  auto sum8 = [&](int c, float(&v)[8]) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = 0.f;
    const YT* src = row + c;
    int s = 0;
    for (; s + 4 <= S; s += 4, src += 4 * slab_stride) {
      SlabVec8<YT> a[4];
#pragma unroll
      for (int q = 0; q < 4; ++q) a[q].load(src + q * slab_stride);
#pragma unroll
      for (int q = 0; q < 4; ++q) a[q].add_to(v);
    }
    for (; s < S; ++s, src += slab_stride) {
      SlabVec8<YT> a;
      a.load(src);
      a.add_to(v);
    }
  };
  auto put8 = [](CT* p, const float(&v)[8]) {
    if constexpr (sizeof(CT) == 2) {
      *reinterpret_cast<u32x4*>(p) = pack8(v);
    } else {
      *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
      *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
    }
  };
  if (tid < 64) {
    const int64_t slot = slots[t];
    if (slot < 0 || !cache) return;
    float ss = 0.f;
    for (int c = tid * 8; c < R; c += 512) {  // columns past `rank` are exact zeros
      float v[8];
      if (ROPE && c >= rope.c_at) break;
      sum8(q_cols + c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)rank + eps);
    CT* out = cache + (size_t)slot * R;
    for (int c = tid * 8; c < R; c += 512) {
      float v[8];
      sum8(q_cols + c, v);
      if (ROPE && c >= rope.c_at) {
        if (c < rope.c_at + rot8) rotate(c - rope.c_at, v);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] *= inv * gain[c + j];
      }
      put8(out + c, v);
    }
  } else if (q_out) {
    for (int c = (tid - 64) * 8; c < q_cols; c += 192 * 8) {
      float v[8];
      sum8(c, v);
      if constexpr (ROPE) {
        const int d = c % rope.D - rope.q_at;
        if (d >= 0 && d < rot8) rotate(d, v);
      }
      put8(q_out + (size_t)t * q_cols + c, v);
    }
  }
}

int latent_write(const void* y, int y_f32, int S, long slab_stride, long ld, void* q_out, int q_cols, const float* gain,
                 void* cache, int cache_f32, const int64_t* slots, int T, int R, int rank, float eps, LatentRope rope,
                 hipStream_t s) {
  if (T <= 0) return 0;
  if (rope.rot && (!q_out || !cache || !rope.freq || !rope.positions || rope.rot < 0 || rope.rot % 2 || rope.D < 8 || rope.D % 8 ||
                   rope.q_at % 8 || rope.c_at % 8 || rope.q_at + rope.rot > rope.D || rope.c_at < rank || q_cols % rope.D ||
                   rope.c_at + rope.rot > R || rope.rot > 4096))
    return hipErrorInvalidValue;
  if (S < 1 || ld % 8 || q_cols % 8 || (cache && (R % 8 || rank < 1 || rank > R || !gain || !slots)) || !slots)
    return hipErrorInvalidValue;
  if (cache_f32 && !y_f32) return hipErrorInvalidValue;
#define DAB_LW1(YT, CT, RO)                                                                                        \
  hipLaunchKernelGGL((latent_write_kernel<YT, CT, RO>), dim3(T), dim3(256), RO ? (rope.rot + 7) / 8 * 32 : 0, s,   \
                     (const YT*)y, S, slab_stride, ld, (CT*)q_out, q_cols, gain, (CT*)cache, slots, R, rank, eps, rope)
#define DAB_LW(YT, CT)                    \
  do {                                    \
    if (rope.rot) DAB_LW1(YT, CT, true);  \
    else DAB_LW1(YT, CT, false);          \
  } while (0)
  if (y_f32 && cache_f32) DAB_LW(float, float);
  else if (y_f32) DAB_LW(float, bf16);
  else DAB_LW(bf16, bf16);
#undef DAB_LW
#undef DAB_LW1
  return hipGetLastError();
}

// --------------------------------------------------------------------------------- latent_gather

// Row i of `out` = the cached latent of packed context row i: sequence b with cu_k[b] <= i < cu_k[b+1],
// token ctx[b] - (cu_k[b+1] - cu_k[b]) + i - cu_k[b] (the tail of its context).  `units` 16-B chunks a row.
__global__ __launch_bounds__(256) void latent_gather_kernel(u32x4* __restrict__ out, const u32x4* __restrict__ cache,
                                                            const int* __restrict__ block_tables, int max_blocks,
                                                            int block_size, const int* __restrict__ cu_k,
                                                            const int* __restrict__ ctx, int B, int total, int units) {
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (i >= total) return;
  int lo = 0, hi = B - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu_k[mid] <= i) lo = mid;
    else hi = mid - 1;
  }
  const int pos = ctx[lo] - cu_k[lo + 1] + i;
  const int blk = block_tables[(size_t)lo * max_blocks + pos / block_size];
  const u32x4* src = cache + ((size_t)blk * block_size + pos % block_size) * units;
  for (int c = lane; c < units; c += 64) out[(size_t)i * units + c] = src[c];
}

int latent_gather(void* out, const void* cache, const int* block_tables, int max_blocks, int block_size,
                  const int* cu_k, const int* ctx, int B, int total, int row_bytes, hipStream_t s) {
  if (total <= 0) return 0;
  if (B < 1 || row_bytes % 16 || block_size < 1) return hipErrorInvalidValue;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((total + 3) / 4), dim3(256), 0, s, (u32x4*)out, (const u32x4*)cache,
                     block_tables, max_blocks, block_size, cu_k, ctx, B, total, row_bytes / 16);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------- latent_key_fill

// K[i, h, q_at + j] = rows[i, c_at + j] for j < 8 units; one 16-B chunk a thread
__global__ __launch_bounds__(256) void latent_key_fill_kernel(bf16* __restrict__ k, long k_tok, int D, const bf16* __restrict__ rows,
                                                              int R, int q_at, int c_at, int units, int H, long total) {
  const long e = (long)blockIdx.x * 256 + threadIdx.x;
  if (e >= total) return;
  const long i = e / (H * units);
  const int r = (int)(e - i * H * units), h = r / units, u = r % units;
  *reinterpret_cast<u32x4*>(k + i * k_tok + (long)h * D + q_at + 8 * u) =
      *reinterpret_cast<const u32x4*>(rows + i * R + c_at + 8 * u);
}

int latent_key_fill(void* k, long k_tok, int D, const void* rows, int R, int q_at, int c_at, int rot, int H, int T, hipStream_t s) {
  if (T <= 0) return 0;
  const int units = (rot + 7) / 8;
  if (rot < 1 || H < 1 || q_at % 8 || c_at % 8 || D % 8 || R % 8 || k_tok % 8 || q_at + 8 * units > D || c_at + 8 * units > R)
    return hipErrorInvalidValue;
  const long total = (long)T * H * units;
  if (total > (1l << 38)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(latent_key_fill_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, s, (bf16*)k, k_tok, D,
                     (const bf16*)rows, R, q_at, c_at, units, H, total);
  return hipGetLastError();
}

// -------------------------------------------------------------------------------------- head_gemm

// Y[t, h, n] = sum_k X[t, h, k] W[row0 + h N + n, k]; W in the fragment layout [rows/16][K/32][64 lanes][8],
// so a wave's weight fragment is one coalesced 1-KB load.  A wave computes 16 NB output columns of one head
// for 16 MI tokens (NB weight and MI token fragments feed NB MI MFMAs); KSPLIT: the 4 waves of a workgroup
// share one such tile, a quarter of K each (wide latents: a short chain of loads per wave instead of
// K / 32), summed through LDS.
template <int MI, int NB, bool KSPLIT>
__global__ __launch_bounds__(256) void head_gemm_kernel(bf16* __restrict__ y, long y_tok, long y_head,
                                                        const bf16* __restrict__ x, long x_tok, long x_head,
                                                        const bf16* __restrict__ w, int row0, int T, int N, int K) {
  __shared__ f32x4 red[KSPLIT ? 4 * MI * NB * 64 : 1];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, g = lane >> 4, li = lane & 15;
  const int nb = (KSPLIT ? blockIdx.x : blockIdx.x * 4 + wave) * NB, h = blockIdx.y, t0 = blockIdx.z * 16 * MI;
  if (nb * 16 >= N) return;
  const int nk = K / 32, kn = KSPLIT ? nk / 4 : nk, kb = KSPLIT ? wave * kn : 0;
  const bf16* wp = w + (((size_t)(row0 + h * N) / 16 + nb) * nk + kb) * 512 + lane * 8;
  const bf16* xp[MI];
#pragma unroll
  for (int i = 0; i < MI; ++i)
    xp[i] = x + (size_t)min(t0 + 16 * i + li, T - 1) * x_tok + (size_t)h * x_head + 32 * kb + 8 * g;
  f32x4 acc[MI][NB];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < NB; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < kn; ++k) {
    bf16x8 a[NB];
#pragma unroll
    for (int j = 0; j < NB; ++j) a[j] = *reinterpret_cast<const bf16x8*>(wp + ((size_t)j * nk + k) * 512);
#pragma unroll
    for (int i = 0; i < MI; ++i) {
      const bf16x8 b = *reinterpret_cast<const bf16x8*>(xp[i] + 32 * k);
#pragma unroll
      for (int j = 0; j < NB; ++j) acc[i][j] = mfma16(a[j], b, acc[i][j]);
    }
  }
  auto store = [&](int i, int j, int ln, const f32x4& v4) {
    const int t = t0 + 16 * i + (ln & 15);
    if (t >= T) return;
    u32x2 v;
    v[0] = pack2bf(v4[0], v4[1]);
    v[1] = pack2bf(v4[2], v4[3]);
    *reinterpret_cast<u32x2*>(y + (size_t)t * y_tok + (size_t)h * y_head + 16 * (nb + j) + 4 * (ln >> 4)) = v;
  };
  if constexpr (KSPLIT) {
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
      for (int j = 0; j < NB; ++j) red[((wave * MI + i) * NB + j) * 64 + lane] = acc[i][j];
    __syncthreads();
    for (int e = threadIdx.x; e < MI * NB * 64; e += 256) {
      f32x4 v = red[e];
#pragma unroll
      for (int s = 1; s < 4; ++s) v += red[s * MI * NB * 64 + e];
      store(e / (64 * NB), (e >> 6) % NB, e & 63, v);
    }
  } else {
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
      for (int j = 0; j < NB; ++j) store(i, j, lane, acc[i][j]);
  }
}

int head_gemm(void* y, long y_tok, long y_head, const void* x, long x_tok, long x_head, const void* w, int row0, int T,
              int H, int N, int K, hipStream_t s) {
  if (T <= 0) return 0;
  if (H < 1 || N % 16 || K % 32 || row0 % 16 || x_tok % 8 || x_head % 8 || y_tok % 4 || y_head % 4 || H > 65535)
    return hipErrorInvalidValue;
  const bool ks = K % 128 == 0 && K >= 256;
#define DAB_HG1(MI, NB, KS)                                                                                       \
  hipLaunchKernelGGL((head_gemm_kernel<MI, NB, KS>),                                                              \
                     dim3(KS ? N / (16 * NB) : (N / (16 * NB) + 3) / 4, H, (T + 16 * MI - 1) / (16 * MI)), dim3(256), 0, \
                     s, (bf16*)y, y_tok, y_head, (const bf16*)x, x_tok, x_head, (const bf16*)w, row0, T, N, K)
#define DAB_HG(MI, NB)               \
  do {                               \
    if (ks) DAB_HG1(MI, NB, true);   \
    else DAB_HG1(MI, NB, false);     \
  } while (0)
  // few tokens: one column block per wave (latency, more workgroups); many: 64 columns per wave
  if (T <= 16) DAB_HG(1, 1);
  else if (T <= 48 || N % 64) DAB_HG(2, 1);
  else if (T <= 128) DAB_HG(1, 4);
  else DAB_HG(2, 4);
#undef DAB_HG
#undef DAB_HG1
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------- latent_decode
// One workgroup (4 waves) = one key partition of one sequence for 16 HT heads.  Each 64-key tile of the
// cache arrives once by LDS-DMA (buffer_load ... lds, non-temporal) and serves both products:
//   S^T = C Q'^T  : wave w computes head tile w % HT for the 16-key sub-tiles w / HT, + 4 / HT, ...;
//                   the fp32 scores go to LDS;
//   softmax       : every wave redoes the (cheap) softmax of all HT head tiles from those scores, so its
//                   probabilities are born in the B-operand layout and no maximum is exchanged;
//   O^T += C^T P^T: wave w owns columns [w VR/4, (w+1) VR/4) of the latent part (the row without a rotated key, which has
//                   no value) of every head tile; C^T fragments by
//                   ds_read_b64_tr_b16 from the same tile.
// One tile buffer per workgroup and two workgroups per CU: one streams while the other computes (a second
// buffer per workgroup was no faster: a tile's math, not its copy, is the chain).  The
// running maximum starts at the sink (its share of the denominator is 1), in partition 0 only.
//
// A sequence's visible keys are split into `parts` equal partitions of whole tiles (at least `min_part`
// keys each), so the split is balanced at every context length; latent_combine merges them.

struct LatentDecodeParams {
  const bf16* q;      // [B, H, R] absorbed queries
  const bf16* cache;  // [num_blocks, block_size, R]
  const int* block_tables;
  int max_blocks, block_size;
  const int* ctx_lens;
  const float* sink;  // [H], or null
  bf16* out;          // [B, H, VR]
  float* part_o;      // [B, H, parts, VR] un-normalised
  float* part_ml;     // [B, H, parts, 2] maximum (log2 domain), denominator
  const int* order;
  int H, groups, window, parts, min_part;
  float scale_log2;
};

constexpr int kLatTile = 64;

// [first visible key, partition origin (tile-aligned), keys per partition, live partitions] of a context
struct LatentSplit {
  int lo, base, len, np;
  __device__ __forceinline__ LatentSplit(int ctx, int window, int parts, int min_part) {
    lo = window > 0 && ctx > window ? ctx - window : 0;
    base = lo & ~(kLatTile - 1);
    const int tiles = (ctx - base + kLatTile - 1) / kLatTile;
    len = max((tiles + parts - 1) / parts * kLatTile, min_part);
    np = (tiles * kLatTile + len - 1) / len;
  }
};

template <int R>
__device__ __forceinline__ int lat_swz(int r) {  // 16-B chunk XOR of tile row r
  return (2 * r) & (R % 128 == 0 ? 15 : 7);
}

template <int R>
__device__ __forceinline__ int lat_off(int r, int c) {  // byte offset of 16-B chunk c of tile row r
  return r * R * 2 + 16 * (c ^ lat_swz<R>(r));
}

template <int R, int VR, int HT>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(LatentDecodeParams p) {
  constexpr int KT = kLatTile, NKK = R / 32, NT = VR / 64, CPR = R / 8;
  constexpr int NKG = 4 / HT, NS = 4 / NKG;        // waves per head tile, 16-key sub-tiles a wave scores
  constexpr int SROW = KT;                         // floats per head row of the score buffer; 16-B chunk c of row r is at c ^ r % 16
  constexpr int TILE = KT * R * 2, PIECES = TILE / 4096;  // 1-KB DMA pieces per wave and tile
  __shared__ __attribute__((aligned(16))) char smem[TILE + 16 * HT * SROW * 4];
  float* sbuf = reinterpret_cast<float*>(smem + TILE);

  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, li = lane & 15;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int part = blockIdx.y, bg = blockIdx.x;
  const int hg = bg % p.groups, b = p.order ? p.order[bg / p.groups] : bg / p.groups;
  const int ctx = p.ctx_lens[b];
  const LatentSplit sp(ctx, p.window, p.parts, p.min_part);
  if (part >= sp.np) return;
  const int k_begin = sp.base + part * sp.len;
  const int k_end = min(ctx, k_begin + sp.len);
  const int h0 = hg * 16 * HT;
  const int ht = w % HT, kg = w / HT;

  const int* bt = p.block_tables + (size_t)b * p.max_blocks;
  auto dma = [&](int k0, int blk) {  // rows past the context read as zeros (descriptor range), masked below
    const bf16* src = p.cache + ((size_t)blk * p.block_size + k0 % p.block_size) * R;
    const auto rs = __builtin_amdgcn_make_buffer_rsrc((void*)src, 0, min(KT, ctx - k0) * R * 2, 0x00020000);
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int piece = i * 4 + w;
      unsigned off;
      int base = 0;
      if constexpr (64 % CPR == 0) {  // whole rows per piece: the lane part repeats every other piece
        const int row = (i & 1) * 4 * (64 / CPR) + w * (64 / CPR) + lane / CPR;
        off = (unsigned)((lane / CPR) * R * 2 + 16 * ((lane % CPR) ^ lat_swz<R>(row)));
        base = piece * 1024;
      } else {
        const int c = piece * 64 + lane, row = c / CPR;
        off = (unsigned)(row * R * 2 + 16 * ((c % CPR) ^ lat_swz<R>(row)));
      }
      __builtin_amdgcn_raw_ptr_buffer_load_lds(rs, (__attribute__((address_space(3))) void*)(smem + piece * 1024), 16,
                                               off, base, 0, 2);
    }
  };
  dma(k_begin, bt[k_begin / p.block_size]);

  bf16x8 qf[NKK];
  {
    const int h = h0 + 16 * ht + li;
    const bool qv = h < p.H;
    const bf16* qrow = p.q + ((size_t)b * p.H + (qv ? h : 0)) * R;
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) {
      bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      qf[kk] = qv ? *reinterpret_cast<const bf16x8*>(qrow + 32 * kk + 8 * g) : z;
    }
  }
  f32x4 o[HT][NT];
  float m_run[HT], l_run[HT];
#pragma unroll
  for (int i = 0; i < HT; ++i) {
#pragma unroll
    for (int t = 0; t < NT; ++t) o[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    m_run[i] = -1e30f;
    l_run[i] = 0.f;
    if (p.sink && part == 0) {
      m_run[i] = p.sink[min(h0 + 16 * i + li, p.H - 1)] * 1.4426950408889634f;
      l_run[i] = g == 0 ? 1.f : 0.f;
    }
  }

  // fragment addresses: the swizzle only permutes chunks inside SW-chunk groups, so a few lane-dependent
  // bases plus instruction offsets reach every fragment
  constexpr int SW = R % 128 == 0 ? 16 : 8, KV = SW / 4;
  const int qq = li >> 2, pp = li & 3;
  int ka[KV];
#pragma unroll
  for (int j = 0; j < KV; ++j) ka[j] = (16 * kg + li) * R * 2 + 16 * ((4 * j + g) ^ lat_swz<R>(li));
  int va[4], vb[4];  // (R % 256 == 0) rows 8 g + qq and + 4 of the wave's first columns
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int in8 = 16 * ((2 * j + (pp >> 1)) ^ (2 * qq)) + 8 * (pp & 1) + (8 * g + qq) * R * 2;
    va[j] = in8 + 128 * w * (CPR / 32);
    vb[j] = in8 + 128 * (R == 256 ? w ^ 1 : w * (CPR / 32)) + 4 * R * 2;
  }
  for (int k0 = k_begin; k0 < k_end; k0 += KT) {
    const int blk = bt[min(k0 + KT, k_end - 1) / p.block_size];  // the next tile's, fetched under this tile's copy
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int sub = kg + NKG * i;
      f32x4 s0 = f32x4{0.f, 0.f, 0.f, 0.f}, s1 = s0;  // two chains: half the MFMA latency
#pragma unroll
      for (int kk = 0; kk < NKK; kk += 2) {
        const char* kp = smem + NKG * i * 16 * R * 2 + SW * 16 * (kk / KV);
        s0 = mfma16(*reinterpret_cast<const bf16x8*>(kp + ka[kk % KV]), qf[kk], s0);
        s1 = mfma16(*reinterpret_cast<const bf16x8*>(kp + ka[kk % KV + 1]), qf[kk + 1], s1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = k0 + 16 * sub + 4 * g + r;
        s0[r] = key >= sp.lo && key < k_end ? (s0[r] + s1[r]) * p.scale_log2 : -__builtin_huge_valf();
      }
      *reinterpret_cast<f32x4*>(sbuf + (16 * ht + li) * SROW + 4 * ((4 * sub + g) ^ li)) = s0;
    }
    __syncthreads();
    bf16x8 pf[HT][2];
#pragma unroll
    for (int i = 0; i < HT; ++i) {
      const float* srow = sbuf + (16 * i + li) * SROW;
      float e[16];
      float mx = -__builtin_huge_valf();
#pragma unroll
      for (int j = 0; j < 4; ++j) {  // keys 32 (j / 2) + 8 g + 4 (j % 2) .. + 4
        const f32x4 v = *reinterpret_cast<const f32x4*>(srow + 4 * ((8 * (j >> 1) + 2 * g + (j & 1)) ^ li));
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          e[4 * j + r] = v[r];
          mx = fmaxf(mx, v[r]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float m_new = fmaxf(m_run[i], mx);
      const float alpha = __builtin_amdgcn_exp2f(m_run[i] - m_new);
      m_run[i] = m_new;
      float ls = 0.f;
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        e[j] = __builtin_amdgcn_exp2f(e[j] - m_new);
        ls += e[j];
      }
      l_run[i] = l_run[i] * alpha + ls;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        u32x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = pack2bf(e[8 * ks + 2 * j], e[8 * ks + 2 * j + 1]);
        pf[i][ks] = __builtin_bit_cast(bf16x8, v);
      }
      if (!__all(alpha == 1.f)) {
#pragma unroll
        for (int t = 0; t < NT; ++t) o[i][t] *= alpha;
      }
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const char *pl, *ph;
        if constexpr (R % 256 == 0 && VR == R) {  // (rows + 4 flip bit 3 of the chunk: the neighbouring 8-chunk group)
          pl = smem + va[t & 3] + 32 * ks * R * 2 + 128 * (t >> 2);
          ph = smem + vb[t & 3] + 32 * ks * R * 2 + (R == 256 ? 0 : 128 * ((t >> 2) ^ 1));
        } else {
          const int ch = w * (VR / 32) + 2 * t + (pp >> 1), row = 32 * ks + 8 * g + qq;
          pl = smem + lat_off<R>(row, ch) + 8 * (pp & 1);
          ph = smem + lat_off<R>(row + 4, ch) + 8 * (pp & 1);
        }
        const bf16x4 lo = ds_read_tr16(pl), hi = ds_read_tr16(ph);
        const bf16x8 a = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
        for (int i = 0; i < HT; ++i) o[i][t] = mfma16(a, pf[i][ks], o[i][t]);
      }
    __syncthreads();  // every wave is done with the tile
    if (k0 + KT < k_end) dma(k0 + KT, blk);
  }

  const size_t hrow = (size_t)b * p.H;
#pragma unroll
  for (int i = 0; i < HT; ++i) {
    const int h = h0 + 16 * i + li;
    float L = l_run[i];
    L += __shfl_xor(L, 16, 64);
    L += __shfl_xor(L, 32, 64);
    if (h >= p.H) continue;
    const int col = w * (VR / 4) + 4 * g;
    if (sp.np == 1) {
      const float inv = L > 0.f ? 1.f / L : 0.f;
      bf16* orow = p.out + (hrow + h) * VR + col;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        u32x2 v;
        v[0] = pack2bf(o[i][t][0] * inv, o[i][t][1] * inv);
        v[1] = pack2bf(o[i][t][2] * inv, o[i][t][3] * inv);
        *reinterpret_cast<u32x2*>(orow + 16 * t) = v;
      }
    } else {
      const size_t pi = (hrow + h) * p.parts + part;
#pragma unroll
      for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(p.part_o + pi * VR + col + 16 * t) = o[i][t];
      if (w == 0 && g == 0) {
        p.part_ml[2 * pi] = m_run[i];
        p.part_ml[2 * pi + 1] = L;
      }
    }
  }
}

// One (sequence, head) per workgroup, 4 columns a thread: the partitions' outputs weighted by
// 2^(m_i - M) over the common denominator.  Sequences with one partition were written directly.
__global__ __launch_bounds__(128) void latent_combine_kernel(LatentDecodeParams p, int R) {
  const int h = blockIdx.x, b = blockIdx.y, c = threadIdx.x * 4;
  const LatentSplit sp(p.ctx_lens[b], p.window, p.parts, p.min_part);
  if (sp.np == 1) return;
  const size_t hrow = (size_t)b * p.H + h;
  const float* ml = p.part_ml + 2 * hrow * p.parts;
  float M = -1e30f;
  for (int i = threadIdx.x & 63; i < sp.np; i += 64) M = fmaxf(M, ml[2 * i]);
  M = wave_max(M);
  if (c >= R) return;
  const float* po = p.part_o + hrow * p.parts * R + c;
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  float L = 0.f;
#pragma unroll 4
  for (int i = 0; i < sp.np; ++i) {
    const float f = __builtin_amdgcn_exp2f(ml[2 * i] - M);
    L = fmaf(f, ml[2 * i + 1], L);
    const f32x4 v = *reinterpret_cast<const f32x4*>(po + (size_t)i * R);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = fmaf(f, v[j], acc[j]);
  }
  const float inv = L > 0.f ? 1.f / L : 0.f;
  u32x2 v;
  v[0] = pack2bf(acc[0] * inv, acc[1] * inv);
  v[1] = pack2bf(acc[2] * inv, acc[3] * inv);
  *reinterpret_cast<u32x2*>(p.out + hrow * R + c) = v;
}

// Rows (padded) the MFMA decode tiles, and the width of a row's latent part: 320 and 576 end with a rotated key.
int latent_decode_ok(int R) {
  return R == 64 || R == 128 || R == 192 || R == 256 || R == 320 || R == 384 || R == 512 || R == 576;
}
int latent_decode_values(int R) { return R == 320 ? 256 : R == 576 ? 512 : R; }

// 16-head tiles of a workgroup: up to 64 heads share one staged latent tile (32 above R = 192: registers)
static int decode_head_tiles(int H, int R) { return H <= 16 ? 1 : (H <= 32 || R > 192 ? 2 : 4); }

int latent_decode_groups(int H, int R) {
  const int ht = decode_head_tiles(H, R);
  return (H + 16 * ht - 1) / (16 * ht);
}

int latent_decode(const void* q, const void* cache, const int* block_tables, int max_blocks, int block_size,
                  const int* ctx_lens, const float* sink, void* out, float* part_o, float* part_ml, int B, int H, int R,
                  int window, int parts, int min_part, float scale, const int* order, hipStream_t s) {
  if (B <= 0) return 0;
  if (H < 1 || !latent_decode_ok(R) || block_size % 64 || parts < 1 || min_part < 64 || min_part % 64 || B > 65535 ||
      (parts > 1 && (!part_o || !part_ml)))
    return hipErrorInvalidValue;
  LatentDecodeParams p{(const bf16*)q, (const bf16*)cache, block_tables, max_blocks, block_size, ctx_lens, sink,
                       (bf16*)out, part_o, part_ml, order, H, latent_decode_groups(H, R), window, parts, min_part,
                       scale * 1.4426950408889634f};
  const int ht = decode_head_tiles(H, R);
  const dim3 grid(B * p.groups, parts);
#define DAB_LD1(RR, VV, HH) hipLaunchKernelGGL((latent_decode_kernel<RR, VV, HH>), grid, dim3(256), 0, s, p)
#define DAB_LDV(RR, VV)                                \
  case RR:                                             \
    if (ht == 1) DAB_LD1(RR, VV, 1);                   \
    else if (ht == 2) DAB_LD1(RR, VV, 2);              \
    else if constexpr (RR <= 192) DAB_LD1(RR, VV, 4);  \
    break;
#define DAB_LD(RR) DAB_LDV(RR, RR)
  switch (R) {
    DAB_LD(64)
    DAB_LD(128)
    DAB_LD(192)
    DAB_LD(256)
    DAB_LD(384)
    DAB_LD(512)
    DAB_LDV(320, 256)
    DAB_LDV(576, 512)
  }
#undef DAB_LD
#undef DAB_LDV
#undef DAB_LD1
  const int err = hipGetLastError();
  if (err || parts == 1) return err;
  const int VR = latent_decode_values(R);
  hipLaunchKernelGGL(latent_combine_kernel, dim3(H, B), dim3(VR <= 256 ? 64 : 128), 0, s, p, VR);
  return hipGetLastError();
}

// ------------------------------------------------------------------------------------- latent_any

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(bf16* p, float v) { *p = f2bf(v); }

constexpr int kAnyMaxRank = 2048;

// q / out [T, H, R] absorbed; token t is query t - cu_q[b] of sequence b (cu_q null: one query per
// sequence); its keys are the window ending at its own position in the paged cache.
template <typename T>
__global__ __launch_bounds__(256) void latent_any_kernel(T* __restrict__ out, const T* __restrict__ q,
                                                         const T* __restrict__ cache,
                                                         const int* __restrict__ block_tables, int max_blocks,
                                                         int block_size, const int* __restrict__ cu_q,
                                                         const int* __restrict__ ctx_lens, int B,
                                                         const float* __restrict__ sink, int H, int R, int window,
                                                         float scale) {
  __shared__ float qs[kAnyMaxRank];
  __shared__ float ps[256];
  __shared__ long rows[256];
  __shared__ float red[4];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  int b = t, pos;
  if (cu_q) {
    int lo = 0, hi = B - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (cu_q[mid] <= t) lo = mid;
      else hi = mid - 1;
    }
    b = lo;
    pos = ctx_lens[b] - cu_q[b + 1] + t;
  } else {
    pos = ctx_lens[b] - 1;
  }
  const int* bt = block_tables + (size_t)b * max_blocks;
  const T* qrow = q + ((size_t)t * H + h) * R;
  for (int i = tid; i < R; i += 256) qs[i] = to_f(qrow[i]);
  float o[kAnyMaxRank / 256];
#pragma unroll
  for (int i = 0; i < kAnyMaxRank / 256; ++i) o[i] = 0.f;
  float m = sink ? sink[h] : -1e30f, l = sink ? 1.f : 0.f;
  __syncthreads();
  const int k_lo = window > 0 && pos + 1 > window ? pos + 1 - window : 0;
  for (int k0 = k_lo; k0 <= pos; k0 += 256) {
    const int n = min(256, pos + 1 - k0);
    float s = -__builtin_huge_valf();
    if (tid < n) {
      const int key = k0 + tid;
      const long row = ((long)bt[key / block_size] * block_size + key % block_size) * R;
      rows[tid] = row;
      const T* c = cache + row;
      float a = 0.f;
      for (int i = 0; i < R; i += 4)
#pragma unroll
        for (int j = 0; j < 4; ++j) a = fmaf(qs[i + j], to_f(c[i + j]), a);
      s = a * scale;
    }
    float mx = wave_max(s);
    if (lane == 0) red[w] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float m_new = fmaxf(m, mx);
    const float e = tid < n ? expf(s - m_new) : 0.f;
    const float f = expf(m - m_new);
    m = m_new;
    ps[tid] = e;
    __syncthreads();  // red read by all, ps / rows complete
    const float es = wave_sum(e);
    if (lane == 0) red[w] = es;
    __syncthreads();
    l = l * f + (red[0] + red[1] + red[2] + red[3]);
#pragma unroll
    for (int i = 0; i < kAnyMaxRank / 256; ++i) {
      const int r = tid + 256 * i;
      if (r < R) {
        float a = o[i] * f;
        for (int j = 0; j < n; ++j) a = fmaf(ps[j], to_f(cache[rows[j] + r]), a);
        o[i] = a;
      }
    }
    __syncthreads();  // ps / rows / red are rewritten by the next chunk
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int i = 0; i < kAnyMaxRank / 256; ++i) {
    const int r = tid + 256 * i;
    if (r < R) put(out + ((size_t)t * H + h) * R + r, o[i] * inv);
  }
}

int latent_any(void* out, const void* q, const void* cache, int f32, const int* block_tables, int max_blocks,
               int block_size, const int* cu_q, const int* ctx_lens, int B, const float* sink, int T, int H, int R,
               int window, float scale, hipStream_t s) {
  if (T <= 0) return 0;
  if (B < 1 || H < 1 || H > 65535 || R % 4 || R > kAnyMaxRank || block_size < 1) return hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(latent_any_kernel<float>, dim3(T, H), dim3(256), 0, s, (float*)out, (const float*)q,
                       (const float*)cache, block_tables, max_blocks, block_size, cu_q, ctx_lens, B, sink, H, R, window,
                       scale);
  else
    hipLaunchKernelGGL(latent_any_kernel<bf16>, dim3(T, H), dim3(256), 0, s, (bf16*)out, (const bf16*)q,
                       (const bf16*)cache, block_tables, max_blocks, block_size, cu_q, ctx_lens, B, sink, H, R, window,
                       scale);
  return hipGetLastError();
}

}  // namespace dab
