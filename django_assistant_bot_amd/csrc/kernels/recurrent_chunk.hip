// Chunked form of the matrix-state recurrences (recurrent.hip) for bf16 prompt portions: 64 tokens at a time on MFMA.
//
// Within a chunk let G_i = log-decay summed up to token i (inclusive), S0 the state before it, and k, q the unit
// vectors.  The recurrence then is (delta; L = strictly lower triangle)
//     M_ij = beta_i e^(G_i - G_j) k_i.k_j  (j < i)          T = (I + M)^-1
//     R_i  = beta_i (v_i - e^(G_i) S0^T k_i)                U = T R
//     o_i  = e^(G_i) S0^T q_i + sum_{j <= i} e^(G_i - G_j) (q_i.k_j) U_j
//     S    = e^(G_C) S0 + sum_j e^(G_C - G_j) k_j U_j^T
// and for state-space duality T = I, U = beta v.  T and A_ij = e^(G_i - G_j) q_i.k_j do not depend on the state:
//   chunk_prepare   every (chunk, head) at once: products of the bf16 inputs, T by forward substitution
//   chunk_scan      the chunks of a sequence in turn; a wave owns 16 value columns of one head and keeps their state
//                   in accumulator registers
//
// Few sequences leave the chip idle while their chunks wait for each other, so long portions are cut into segments of
// kSeg chunks that run side by side: chunk_scan in its SUMMARY form first computes what a segment does to any state,
// S_end = P S_start + S_loc (delta: P by scanning the columns of the identity without values; ssd: P is the scalar
// e^(G of the segment)), chunk_combine walks the segments with it, and the segments are then scanned from their own
// start states.
//
// Precision: everything is an fp32 computation.  The convolved q, k are exact bf16 numbers, so their products on the
// bf16 MFMA are exact fp32 products; unit-norm factors, decays and betas are fp32 row scales applied outside.  An fp32
// operand X (S, R, U, T) enters as X = hi + mid + lo, three bf16 terms (24 bits): products with a bf16 operand take 3
// MFMAs, fp32 x fp32 the 6 whose weight exceeds 2^-24.  (A, which only reaches the bf16 output, has two terms.)
//
// Operand order: the accumulator layout (lane g = lane / 16 holds rows 4 g + r of a 16-row tile) is fed straight back
// as a B operand by letting k slot (g, j) of a 32-deep step be row 4 g + j of its first tile for j < 4 and row
// 4 g + j - 4 of its second tile otherwise; A operands are read in the same order.
#include "launchers.h"
#include "proj.h"

namespace dab {

namespace {

constexpr int kC = 64;          // tokens of a chunk
constexpr int kPairs = 6;       // (16-row tile, 32-deep step) pairs of a lower-triangular 64 x 64 operand
constexpr int kFrag = 1024;     // bytes of one A fragment
constexpr int kT = kPairs * 3 * kFrag, kA = kPairs * 2 * kFrag, kScal = 2048;  // (5 rows of kC floats used)
constexpr int kWs = kT + kA + kScal;  // workspace of one (chunk, head)

__device__ __forceinline__ int pair_id(int m, int kb) { return m < 2 ? m : 2 + 2 * (m - 2) + kb; }

struct ChunkP {
  const bf16* conv;
  int C, q_col, k_col, v_col;
  int H, G, D, V;
  Proj gates;
  int a_col, b_col;
  const float* A;
  const float* dt_bias;
  const float* skip;
  float* state;
  const int* slot;
  const int* pos;
  const int* cu;
  bf16* out;
  char* ws;
  float qscale;
  int segs;          // segments per sequence (1: whole sequences)
  float* seg_start;  // [chunks, segs, H, V, Dp] state before each segment but a sequence's first
  float* seg_loc;    // [chunks, segs, H, V (+ Dp), Dp] summaries
};

constexpr int kSeg = 16;  // chunks of a segment

// x = hi + mid (+ lo), bf16 each
template <int N>
__device__ __forceinline__ void split(const float (&x)[8], bf16x8 (&o)[N]) {
  float r[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) r[j] = x[j];
#pragma unroll
  for (int n = 0; n < N; ++n) {
    u32x4 p;
#pragma unroll
    for (int j = 0; j < 4; ++j) p[j] = pack2bf(r[2 * j], r[2 * j + 1]);
    o[n] = __builtin_bit_cast(bf16x8, p);
    if (n + 1 < N) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        r[2 * j] -= __uint_as_float(p[j] << 16);
        r[2 * j + 1] -= __uint_as_float(p[j] & 0xffff0000u);
      }
    }
  }
}

__device__ __forceinline__ bf16x8 cat4(const bf16x4& a, const bf16x4& b) {
  return bf16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// The K | Q tile of a chunk, 16-B pieces e = tid + 256 i.  Loads are unconditional (a load behind a lane mask waits for
// its data on the spot): rows past the portion repeat its last one, which zero betas and triangles keep out of every
// result; columns past D become zeros.
template <int D32>
constexpr int kPieces = 2 * kC * 4 * D32 / 256;

template <int D32>
__device__ __forceinline__ void fetch_kq(const ChunkP& p, int row, int n, int hk, int tid, u32x4 (&pre)[kPieces<D32>]) {
  constexpr int PR = 4 * D32;
#pragma unroll
  for (int i = 0; i < kPieces<D32>; ++i) {
    const int e = tid + 256 * i, t = min(e / PR % kC, n - 1), ch = e % PR;
    const int c = min(ch * 8, p.D - 8) + (e >= kC * PR ? p.q_col : p.k_col) + hk * p.D;
    pre[i] = *reinterpret_cast<const u32x4*>(p.conv + (size_t)(row + t) * p.C + c);
    if (ch * 8 >= p.D) pre[i] = u32x4{0, 0, 0, 0};
  }
}

template <int D32>
__device__ __forceinline__ void store_kq(char* lds, int tid, const u32x4 (&pre)[kPieces<D32>]) {
  constexpr int PR = 4 * D32, STR = 64 * D32 + 16;
#pragma unroll
  for (int i = 0; i < kPieces<D32>; ++i) {
    const int e = tid + 256 * i;
    *reinterpret_cast<u32x4*>(lds + (e >= kC * PR ? kC * STR : 0) + e / PR % kC * STR + e % PR * 16) = pre[i];
  }
}

// ssd: one workgroup per (chunk, q / k group), its products once, then decays and output head by head; delta: one
// workgroup per (chunk, head), whose triangular solve is the longer part.
template <int D32, bool DELTA>
__global__ __launch_bounds__(256) void chunk_prepare_kernel(ChunkP p) {
  constexpr int Dp = 32 * D32, STR = Dp * 2 + 16, LD = 68;
  constexpr int KQ = 2 * kC * STR, MA = (DELTA ? 2 : 1) * kC * LD * 4;
  __shared__ __attribute__((aligned(16))) char smem[KQ > MA ? KQ : MA];
  __shared__ double gam[kC];  // sums in fp64: their small differences are what counts
  __shared__ float be[kC], kk[kC], qq[kC];
  char* ks = smem;
  char* qs = smem + kC * STR;
  float* Am = reinterpret_cast<float*>(smem);
  float* Mm = Am + kC * LD;
  const int rep = p.H / p.G;
  const int c = blockIdx.x, hk = DELTA ? blockIdx.y / rep : blockIdx.y, b = blockIdx.z;
  const int h_first = DELTA ? blockIdx.y : hk * rep, h_last = DELTA ? h_first : h_first + rep - 1;
  const int r0 = p.cu[b] + kC * c, n = min(kC, p.cu[b + 1] - r0);
  if (n <= 0) return;
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, g = lane >> 4, li = lane & 15;
  u32x4 pre[kPieces<D32>];
  fetch_kq<D32>(p, r0, n, hk, tid, pre);
  store_kq<D32>(smem, tid, pre);
  if (!DELTA && tid < kC) kk[tid] = qq[tid] = 1.f;
  __syncthreads();
  // rows 16 w .. of K K^T and Q K^T (lower triangle), and the diagonal of Q Q^T
  f32x4 kkt[4], qkt[4], qqt = {0.f, 0.f, 0.f, 0.f};
  bf16x8 ka[D32], qa[D32];
#pragma unroll
  for (int kb = 0; kb < D32; ++kb) {
    ka[kb] = *reinterpret_cast<const bf16x8*>(ks + (16 * w + li) * STR + (32 * kb + 8 * g) * 2);
    qa[kb] = *reinterpret_cast<const bf16x8*>(qs + (16 * w + li) * STR + (32 * kb + 8 * g) * 2);
    if (DELTA) qqt = mfma16(qa[kb], qa[kb], qqt);
  }
#pragma unroll
  for (int nt = 0; nt < 4; ++nt) {
    kkt[nt] = qkt[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (nt > w) continue;
#pragma unroll
    for (int kb = 0; kb < D32; ++kb) {
      const bf16x8 kn = *reinterpret_cast<const bf16x8*>(ks + (16 * nt + li) * STR + (32 * kb + 8 * g) * 2);
      if (DELTA) kkt[nt] = mfma16(ka[kb], kn, kkt[nt]);
      qkt[nt] = mfma16(qa[kb], kn, qkt[nt]);
    }
    if (DELTA && nt == w) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (4 * g + r == li) {
          kk[16 * w + li] = 1.f / sqrtf(kkt[nt][r] + 1e-6f);
          qq[16 * w + li] = p.qscale / sqrtf(qqt[r] + 1e-6f);
        }
    }
  }
  auto frag = [&](const float* src, int m, int kb, float(&x)[8]) {
    const float* s = src + (16 * m + li) * LD + 32 * kb + 4 * g;
    const f32x4 lo = *reinterpret_cast<const f32x4*>(s), hi = *reinterpret_cast<const f32x4*>(s + 16);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      x[j] = lo[j];
      x[4 + j] = hi[j];
    }
  };
  auto row_of = [](int pr) { return pr < 2 ? pr : 2 + (pr - 2) / 2; };
  auto step_of = [](int pr) { return pr < 2 ? 0 : (pr - 2) % 2; };
  for (int h = h_first; h <= h_last; ++h) {
    char* ws = p.ws + ((size_t)(p.cu[b] / kC + b + c) * p.H + h) * kWs;
    __syncthreads();  // K / Q, or the previous head's matrices, are done with
    if (w == 0) {
      float beta = 0.f;
      double dl = 0.;
      if (lane < n) {
        const float z = proj_f32<float>(p.gates, r0 + lane, p.a_col + h) + p.dt_bias[h];
        const float dt = z > 20.f ? z : log1pf(__expf(z));
        dl = -p.A[h] * dt;
        beta = DELTA ? 1.f / (1.f + __expf(-proj_f32<float>(p.gates, r0 + lane, p.b_col + h))) : dt;
      }
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double x = __shfl_up(dl, o, 64);
        if (lane >= o) dl += x;
      }
      gam[lane] = dl;
      be[lane] = beta;
    }
    __syncthreads();
#pragma unroll
    for (int nt = 0; nt < 4; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * w + 4 * g + r, j = 16 * nt + li;
        float m = 0.f, a = 0.f;
        if (j <= i) {
          const float e = __expf((float)(gam[i] - gam[j])) * kk[j];
          a = e * qq[i] * qkt[nt][r];
          if (DELTA && j < i) m = be[i] * e * kk[i] * kkt[nt][r];
        }
        if (DELTA) Mm[i * LD + j] = m;
        Am[i * LD + j] = a;
      }
    __syncthreads();
    if (w == 0) {
      float* sc = reinterpret_cast<float*>(ws + kT + kA);
      const float eg = __expf((float)gam[lane]);
      sc[lane] = be[lane];
      sc[kC + lane] = eg * kk[lane];
      sc[2 * kC + lane] = eg * qq[lane];
      sc[3 * kC + lane] = __expf((float)(gam[kC - 1] - gam[lane])) * kk[lane];
      sc[4 * kC + lane] = eg;
      if (DELTA) {
        // column ``lane`` of T: t_i = [i == lane] - sum_{j < i} M_ij t_j
        float t[kC];
#pragma unroll
        for (int i = 0; i < kC; ++i) {
          float a[4] = {lane == i ? 1.f : 0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
            const f32x4 mv = *reinterpret_cast<const f32x4*>(Mm + i * LD + 4 * j4);
#pragma unroll
            for (int q = 0; q < 4; ++q)
              if (4 * j4 + q < i) a[q] = fmaf(-mv[q], t[4 * j4 + q], a[q]);
          }
          t[i] = (a[0] + a[1]) + (a[2] + a[3]);
        }
#pragma unroll
        for (int i = 0; i < kC; ++i) Mm[i * LD + lane] = t[i];  // every read of M was this wave's own
      }
    }
    if (w > 0 || !DELTA)
      for (int pr = DELTA ? w - 1 : w; pr < kPairs; pr += DELTA ? 3 : 4) {
        float x[8];
        bf16x8 o[2];
        frag(Am, row_of(pr), step_of(pr), x);
        split(x, o);
#pragma unroll
        for (int s = 0; s < 2; ++s) *reinterpret_cast<bf16x8*>(ws + kT + (2 * pr + s) * kFrag + lane * 16) = o[s];
      }
    if constexpr (!DELTA) continue;
    __syncthreads();
    for (int pr = w; pr < kPairs; pr += 4) {
      float x[8];
      bf16x8 o[3];
      frag(Mm, row_of(pr), step_of(pr), x);
      split(x, o);
#pragma unroll
      for (int s = 0; s < 3; ++s) *reinterpret_cast<bf16x8*>(ws + (3 * pr + s) * kFrag + lane * 16) = o[s];
    }
  }
}

// LDS: the chunk's K | Q tile (rows prefetched into registers a chunk ahead) and its workspace block (T and A fragments,
// row scales), copied by LDS-DMA as soon as every wave is done with the previous one.
template <int D32, bool DELTA, bool SUMMARY>
__global__ __launch_bounds__(256, 2) void chunk_scan_kernel(ChunkP p) {
  constexpr int Dp = 32 * D32, STR = Dp * 2 + 16, MT = 2 * D32;
  constexpr int P0 = DELTA ? 0 : kT / 1024, P1 = kWs / 1024;  // 1-KB pieces of the workspace block that are needed
  __shared__ __attribute__((aligned(16))) char smem[2 * kC * STR + kWs];
  char* const ks = smem;
  char* const qs = smem + kC * STR;
  char* const wl = smem + 2 * kC * STR;
  const float* const sc = reinterpret_cast<const float*>(wl + kT + kA);  // beta, e^G k-norm, e^G q-norm, e^(G_C - G) k-norm, e^G
  const int h = blockIdx.y, b = blockIdx.z / p.segs, seg = blockIdx.z % p.segs, hk = h / (p.H / p.G);
  const int q0 = p.cu[b], len = p.cu[b + 1] - q0;
  const int nca = (len + kC - 1) / kC;  // chunks of the portion; this workgroup's are c0 .. nc - 1
  const int c0 = p.segs > 1 ? seg * kSeg : 0, nc = p.segs > 1 ? min(nca, c0 + kSeg) : nca;
  if (c0 >= nca || (SUMMARY && nc == nca)) return;  // (nothing needs the last segment's summary)
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, li = lane & 15;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int vb = (p.V + 63) / 64;
  const bool ident = SUMMARY && (int)blockIdx.x >= vb;  // columns of the identity
  const int ncol = ident ? Dp : p.V, bx = ident ? blockIdx.x - vb : blockIdx.x;
  const int col = bx * 64 + 16 * w + li;
  const bool live = bx * 64 + 16 * w < ncol, mine = col < ncol;
  const size_t bs = (size_t)(b * p.segs + seg) * p.H + h;
  float* const slot_state = p.state + (((size_t)p.slot[b] * p.H + h) * p.V + (mine ? col : 0)) * Dp + 4 * g;
  const float* sp = seg > 0 ? p.seg_start + (bs * p.V + (mine ? col : 0)) * Dp + 4 * g : slot_state;
  const char* ws0 = p.ws + ((size_t)(q0 / kC + b) * p.H + h) * kWs;
  f32x4 S[MT];
  const bool fresh = SUMMARY || !mine || (seg == 0 && p.pos[q0] == 0);
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    S[m] = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(sp + 16 * m);
    if (SUMMARY && ident) {
#pragma unroll
      for (int r = 0; r < 4; ++r) S[m][r] = 16 * m + 4 * g + r == col ? 1.f : 0.f;
    }
  }
  const float skip = !DELTA && p.skip ? p.skip[h] : 0.f;
  u32x4 pre[kPieces<D32>];
  auto fetch = [&](int c) { fetch_kq<D32>(p, q0 + kC * c, min(kC, len - kC * c), hk, tid, pre); };
  auto copy_ws = [&](int c) {
    const char* src = ws0 + (size_t)c * p.H * kWs + lane * 16;
    for (int i = P0 + w; i < P1; i += 4)
      __builtin_amdgcn_global_load_lds((const void*)(src + i * 1024),
                                       (__attribute__((address_space(3))) void*)(wl + i * 1024), 16, 0, 0);
  };
  auto gather8 = [](const f32x4& a, const f32x4& c, float(&x)[8]) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      x[r] = a[r];
      x[4 + r] = c[r];
    }
  };
  auto scale4 = [&](int row, int m) { return *reinterpret_cast<const f32x4*>(sc + row * kC + 16 * m + 4 * g); };
  fetch(c0);
  copy_ws(c0);
  for (int c = c0; c < nc; ++c) {
    const int n = min(kC, len - kC * c);
    __syncthreads();  // the previous chunk's tile is done with
    store_kq<D32>(smem, tid, pre);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's workspace pieces landed
    __syncthreads();
    f32x4 R[4];  // values of this wave's columns in the accumulator layout
    const bf16* vp = p.conv + (size_t)(q0 + kC * c) * p.C + p.v_col + h * p.V + (mine && !ident ? col : 0);
    const float von = ident ? 0.f : 1.f;
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) R[m][r] = von * bf2f(vp[(size_t)min(16 * m + 4 * g + r, n - 1) * p.C]);
    if (c + 1 < nc) fetch(c + 1);
    bf16x8 wu[2][3];
    float ec = 0.f;
    if (live) {
      bf16x8 ss[D32][3];  // the state as three bf16 terms
#pragma unroll
      for (int kb = 0; kb < D32; ++kb) {
        float x[8];
        gather8(S[2 * kb], S[2 * kb + 1], x);
        split(x, ss[kb]);
      }
      auto times_s = [&](const char* src, int m) {  // A operand: 16 token rows, 32 state rows in slot order
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < D32; ++kb) {
          const char* s = src + (16 * m + li) * STR + (32 * kb + 4 * g) * 2;
          const bf16x8 a = cat4(*reinterpret_cast<const bf16x4*>(s), *reinterpret_cast<const bf16x4*>(s + 32));
          acc = mfma16(a, ss[kb][2], acc);
          acc = mfma16(a, ss[kb][1], acc);
          acc = mfma16(a, ss[kb][0], acc);
        }
        return acc;
      };
      f32x4 U[4], O[4];
      if (DELTA) {
        f32x4 P[4];
#pragma unroll
        for (int m = 0; m < 4; ++m) P[m] = times_s(ks, m);
        if (!SUMMARY) {
#pragma unroll
          for (int m = 0; m < 4; ++m) O[m] = times_s(qs, m) * scale4(2, m);
        }
#pragma unroll
        for (int m = 0; m < 4; ++m) R[m] = scale4(0, m) * (R[m] - scale4(1, m) * P[m]);
        bf16x8 rs[2][3];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
          float x[8];
          gather8(R[2 * kb], R[2 * kb + 1], x);
          split(x, rs[kb]);
        }
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int kb = 0; kb <= m / 2; ++kb) {
            const char* f = wl + 3 * pair_id(m, kb) * kFrag + lane * 16;
            const bf16x8 t0 = *reinterpret_cast<const bf16x8*>(f), t1 = *reinterpret_cast<const bf16x8*>(f + kFrag),
                         t2 = *reinterpret_cast<const bf16x8*>(f + 2 * kFrag);
            acc = mfma16(t2, rs[kb][0], acc);
            acc = mfma16(t0, rs[kb][2], acc);
            acc = mfma16(t1, rs[kb][1], acc);
            acc = mfma16(t1, rs[kb][0], acc);
            acc = mfma16(t0, rs[kb][1], acc);
            acc = mfma16(t0, rs[kb][0], acc);
          }
          U[m] = acc;
        }
      } else {
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          if (!SUMMARY) O[m] = times_s(qs, m) * scale4(2, m) + skip * R[m];
          U[m] = scale4(0, m) * R[m];
        }
      }
      if constexpr (!SUMMARY) {  // read-out
      bf16x8 us[2][2];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float x[8];
        gather8(U[2 * kb], U[2 * kb + 1], x);
        split(x, us[kb]);
      }
#pragma unroll
      for (int m = 0; m < 4; ++m) {
#pragma unroll
        for (int kb = 0; kb <= m / 2; ++kb) {
          const char* f = wl + kT + 2 * pair_id(m, kb) * kFrag + lane * 16;
          const bf16x8 a0 = *reinterpret_cast<const bf16x8*>(f), a1 = *reinterpret_cast<const bf16x8*>(f + kFrag);
          O[m] = mfma16(a1, us[kb][0], O[m]);
          O[m] = mfma16(a0, us[kb][1], O[m]);
          O[m] = mfma16(a0, us[kb][0], O[m]);
        }
      }
      if (mine) {
        bf16* op = p.out + (size_t)(q0 + kC * c) * p.H * p.V + h * p.V + col;
        const size_t ld = (size_t)p.H * p.V;
        if (n == kC) {
#pragma unroll
          for (int m = 0; m < 4; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) op[(16 * m + 4 * g + r) * ld] = f2bf(O[m][r]);
        } else {
#pragma unroll
          for (int m = 0; m < 4; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (16 * m + 4 * g + r < n) op[(16 * m + 4 * g + r) * ld] = f2bf(O[m][r]);
        }
      }
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float x[8];
        gather8(U[2 * kb] * scale4(3, 2 * kb), U[2 * kb + 1] * scale4(3, 2 * kb + 1), x);
        split(x, wu[kb]);
      }
      ec = sc[4 * kC + kC - 1];
    }
    __syncthreads();  // every wave is done with the workspace block
    if (c + 1 < nc) copy_ws(c + 1);
    if (live) {
      // state: S = e^(G_C) S + K^T (e^(G_C - G) U)
      const int tq = li >> 2, tp = li & 3;
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        f32x4 acc = S[m] * ec;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
          const bf16x4 lo = ds_read_tr16(ks + (32 * kb + 4 * g + tq) * STR + (16 * m + 4 * tp) * 2);
          const bf16x4 hi = ds_read_tr16(ks + (32 * kb + 16 + 4 * g + tq) * STR + (16 * m + 4 * tp) * 2);
          const bf16x8 a = cat4(lo, hi);
          acc = mfma16(a, wu[kb][2], acc);
          acc = mfma16(a, wu[kb][1], acc);
          acc = mfma16(a, wu[kb][0], acc);
        }
        S[m] = acc;
      }
    }
  }
  if (mine && (SUMMARY || nc == nca)) {
    float* dst = SUMMARY ? p.seg_loc + (bs * (DELTA ? p.V + Dp : p.V) + (ident ? p.V : 0) + col) * Dp + 4 * g : slot_state;
#pragma unroll
    for (int m = 0; m < MT; ++m) *reinterpret_cast<f32x4*>(dst + 16 * m) = S[m];
  }
}

// Start states of a sequence's segments, one after the other; a workgroup owns 16 value columns of one head.
template <int D32, bool DELTA>
__global__ __launch_bounds__(256) void chunk_combine_kernel(ChunkP p) {
  constexpr int Dp = 32 * D32;
  __shared__ __attribute__((aligned(16))) float st[16][Dp];
  const int h = blockIdx.y, b = blockIdx.z, col0 = blockIdx.x * 16;
  const int q0 = p.cu[b], len = p.cu[b + 1] - q0, nca = (len + kC - 1) / kC, ns = (nca + kSeg - 1) / kSeg;
  if (ns < 2) return;
  const int d = threadIdx.x % 128, half = threadIdx.x / 128;  // this thread's state row, and columns 8 half .. + 7
  const bool fresh = p.pos[q0] == 0, on = d < Dp;
  const float* s0 = p.state + ((size_t)p.slot[b] * p.H + h) * p.V * Dp;
  float x[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = min(col0 + 8 * half + i, p.V - 1);
    x[i] = fresh || !on ? 0.f : s0[(size_t)c * Dp + d];
  }
  for (int s = 0; s + 1 < ns; ++s) {
    const size_t bs = (size_t)(b * p.segs + s) * p.H + h;
    const float* loc = p.seg_loc + bs * (DELTA ? p.V + Dp : p.V) * Dp;
    float y[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) y[i] = on ? loc[(size_t)min(col0 + 8 * half + i, p.V - 1) * Dp + d] : 0.f;
    if (DELTA) {
      __syncthreads();
      if (on)
#pragma unroll
        for (int i = 0; i < 8; ++i) st[8 * half + i][d] = x[i];
      __syncthreads();
      const float* P = loc + (size_t)p.V * Dp + (on ? d : 0);
#pragma unroll 2
      for (int j = 0; j < Dp; j += 4) {
        float pc[4];
#pragma unroll
        for (int q = 0; q < 4; ++q) pc[q] = P[(size_t)(j + q) * Dp];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const f32x4 v = *reinterpret_cast<const f32x4*>(&st[8 * half + i][j]);
#pragma unroll
          for (int q = 0; q < 4; ++q) y[i] = fmaf(pc[q], v[q], y[i]);
        }
      }
    } else {
      float gseg = 1.f;
      const char* ws = p.ws + ((size_t)(q0 / kC + b + s * kSeg) * p.H + h) * kWs + kT + kA;
#pragma unroll
      for (int c = 0; c < kSeg; ++c) gseg *= reinterpret_cast<const float*>(ws + (size_t)c * p.H * kWs)[4 * kC + kC - 1];
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] = fmaf(gseg, x[i], y[i]);
    }
    float* nx = p.seg_start + (bs + p.H) * p.V * Dp;  // (segment s + 1)
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] = y[i];
      if (on && col0 + 8 * half + i < p.V) nx[(size_t)(col0 + 8 * half + i) * Dp + d] = y[i];
    }
  }
}

}  // namespace

// Segments per sequence of a launch: 1, unless whole sequences would leave most CUs idle
int state_chunks_segments(RecurrentShape d, int chunks, int max_q) {
  const int nca = (max_q + kC - 1) / kC;
  const long wgs = (long)((d.V + 63) / 64) * d.H * chunks;
  return wgs <= 128 && nca >= 2 * kSeg ? (nca + kSeg - 1) / kSeg : 1;
}

static long seg_floats(RecurrentShape d, int chunks, int segs, bool loc) {
  return segs < 2 ? 0 : (long)chunks * segs * d.H * (d.V + (loc && d.delta ? d.Dp : 0)) * d.Dp;
}

long state_chunks_bytes(RecurrentShape d, int T, int chunks, int segs) {
  return (long)(T / kC + chunks) * d.H * kWs + 4 * (seg_floats(d, chunks, segs, false) + seg_floats(d, chunks, segs, true));
}

int state_chunks_ok(RecurrentShape d) {
  return d.D % 8 == 0 && d.Dp <= 128 && d.C % 8 == 0 && d.q_col % 8 == 0 && d.k_col % 8 == 0 && d.H >= 1 && d.G >= 1 &&
         d.H % d.G == 0 && d.H <= 65535 && d.Dp == recurrent_state_width(d.D);
}

int state_chunks(const void* conv, RecurrentShape d, Proj gates, const float* A, const float* dt_bias, const float* skip,
                 float* state, const int* slot, const int* pos, const int* cu, int chunks, int max_q, int T, int segs, void* out,
                 void* ws, hipStream_t s) {
  if (chunks <= 0 || max_q <= 0) return 0;
  if (!state_chunks_ok(d) || !gates.f32 || gates.S < 1 || segs < 1 || (long)chunks * segs > 65535 || !ws ||
      (segs > 1 && segs < (max_q + kC * kSeg - 1) / (kC * kSeg)))
    return hipErrorInvalidValue;
  ChunkP p{};
  p.conv = (const bf16*)conv;
  p.C = d.C;
  p.q_col = d.q_col;
  p.k_col = d.k_col;
  p.v_col = d.v_col;
  p.H = d.H;
  p.G = d.G;
  p.D = d.D;
  p.V = d.V;
  p.gates = gates;
  p.a_col = d.a_col;
  p.b_col = d.b_col;
  p.A = A;
  p.dt_bias = dt_bias;
  p.skip = skip;
  p.state = state;
  p.slot = slot;
  p.pos = pos;
  p.cu = cu;
  p.out = (bf16*)out;
  p.ws = (char*)ws;
  p.segs = segs;
  p.seg_start = (float*)((char*)ws + (long)(T / kC + chunks) * d.H * kWs);
  p.seg_loc = p.seg_start + seg_floats(d, chunks, segs, false);
  p.qscale = 1.f / sqrtf((float)d.D);
  const int vb = (d.V + 63) / 64;
  const dim3 gp((max_q + kC - 1) / kC, d.delta ? d.H : d.G, chunks), gs(vb, d.H, chunks * segs);
  const dim3 gm(vb + (d.delta ? (d.Dp + 63) / 64 : 0), d.H, chunks * segs), gc((d.V + 15) / 16, d.H, chunks);
#define CHUNK_D(D32, DELTA)                                                                        \
  do {                                                                                             \
    hipLaunchKernelGGL((chunk_prepare_kernel<D32, DELTA>), gp, dim3(256), 0, s, p);                \
    if (segs > 1) {                                                                                \
      hipLaunchKernelGGL((chunk_scan_kernel<D32, DELTA, true>), gm, dim3(256), 0, s, p);           \
      hipLaunchKernelGGL((chunk_combine_kernel<D32, DELTA>), gc, dim3(256), 0, s, p);              \
    }                                                                                              \
    hipLaunchKernelGGL((chunk_scan_kernel<D32, DELTA, false>), gs, dim3(256), 0, s, p);            \
  } while (0)
#define CHUNK_L(D32)                 \
  do {                               \
    if (d.delta) CHUNK_D(D32, true); \
    else CHUNK_D(D32, false);        \
  } while (0)
  switch (d.Dp / 32) {
    case 1: CHUNK_L(1); break;
    case 2: CHUNK_L(2); break;
    case 3: CHUNK_L(3); break;
    case 4: CHUNK_L(4); break;
    default: return hipErrorInvalidValue;
  }
#undef CHUNK_L
#undef CHUNK_D
  return hipGetLastError();
}

}  // namespace dab
