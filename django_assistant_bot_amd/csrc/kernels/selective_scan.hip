// Selective scan (Mamba): a diagonal state of N entries per channel, carried in fp32 from step to step in per-sequence
// slots.  Per channel c and entry n, with step dt_c > 0, input B_n and read-out C_n of the token:
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c u_c B_n;   y_c = (sum_n S[c, n] C_n + D_c u_c) silu(z_c)
// u is the convolved input, dt = softplus(W_dt low + bias), and low | B | C come from one narrow projection of u.
//
//   narrow_rows     slabs of that projection -> fp32 rows, and its first columns in bf16 (operand of W_dt)
//   selective_scan  prompt portions: a workgroup walks one sequence for a block of channels, a tile of tokens at a time
//                   (few long portions are cut into segments that run side by side: each is summed up from a zero state,
//                   selective_combine walks the summaries -- a segment takes S to exp(A sum dt) S + S_loc --, and then
//                   all are scanned from their own start states)
//   selective_step  one decoded token per sequence, the gate's rows being replaced by the result; W_dt low is formed in the kernel on MFMA, for up to 16 sequences at once
//
// A channel is shared by L neighbouring lanes, NS entries each, so a step's read-out is a sum over L lanes; four tokens'
// sums are transposed across a quad, so each lane finishes one of them.  The state is stored [slot][channel][Np], Np = L NS
// (zeros past N); A holds -exp(A_log) log2(e), so a decay is one v_exp.  Everything but u, z and the output is fp32.
#include "launchers.h"
#include "proj.h"

namespace dab {

// values of the lane whose quad index is ^1 / ^2, and of the lane 4 / 8 further in its row of 16
template <int CTRL>
__device__ __forceinline__ float dpp(float v) {
  return __uint_as_float((unsigned)__builtin_amdgcn_update_dpp(0, (int)__float_as_uint(v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float quad_xor1(float v) { return dpp<0xB1>(v); }
__device__ __forceinline__ float quad_xor2(float v) { return dpp<0x4E>(v); }

// sum over the quads of a group of L lanes (each lane's quad index kept)
template <int L>
__device__ __forceinline__ float across_quads(float v) {
  if (L == 8) v += __shfl_xor(v, 4, 64);
  if (L == 16) {
    v += dpp<0x124>(v);  // row_ror:4
    v += dpp<0x128>(v);  // row_ror:8
  }
  return v;
}

int selective_state_width(int N) {
  if (N < 1 || N > 256) return 0;
  return N <= 64 ? (N + 15) / 16 * 16 : N <= 128 ? 128 : 256;
}

// ----------------------------------------------------------------------------------------------

template <bool LOW>
__global__ __launch_bounds__(256) void narrow_rows_kernel(Proj z, float* __restrict__ out, bf16* __restrict__ low, int N, int R,
                                                          long total) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int w = N / 8;
  const long t = i / w;
  const int c = (int)(i - t * w) * 8;
  float v[8];
  proj8<float>(z, t, c, v);
  ElemIO<float>::store8(out + t * N + c, v);
  if (LOW && c < R) ElemIO<bf16>::store8(low + t * R + c, v);
}

int narrow_rows(Proj z, float* out, void* low, int N, int R, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (!z.f32 || z.S < 1 || N < 8 || N % 8 || R % 8 || R > N || z.ld % 4 || z.slab % 4) return hipErrorInvalidValue;
  const long total = (long)T * (N / 8);
  if (total > (1l << 38)) return hipErrorInvalidValue;
  const dim3 grid((unsigned)((total + 255) / 256));
  if (low) hipLaunchKernelGGL(narrow_rows_kernel<true>, grid, dim3(256), 0, s, z, out, (bf16*)low, N, R, total);
  else hipLaunchKernelGGL(narrow_rows_kernel<false>, grid, dim3(256), 0, s, z, out, (bf16*)low, N, R, total);
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------
// prompt portions

struct SelScan {
  const void* u;        // [T, C] convolved input
  SelectiveShape d;
  Proj dt;              // fp32 [T, C]: W_dt low
  Proj bc;              // fp32 rows of the narrow projection (one slab)
  Proj y;               // input projection, gate columns from z_col
  const float* A;       // [C, Np]
  const float* bias;    // [C]
  const float* skip;    // [C]
  float* state;
  const int* slot;
  const int* pos;
  const int* cu;
  void* out;            // [T, C]
  // segments: tokens of one, their number, start states (and before: summaries) [chunks, segs, C, Np], step sums
  // [chunks, segs, C]
  int seg_len, segs;
  float* starts;
  float* sums;
};

enum ScanMode { SCAN_WHOLE, SCAN_SUMMARY, SCAN_SEGMENT };

// A lane holds its NS entries of CPT channels, 256 / L apart, so that a token's B and C are read once for all of them.
template <typename PT, typename AT, int L, int NS, int CPT, int TB, int MODE>
__global__ __launch_bounds__(256) void selective_scan_kernel(SelScan p) {
  constexpr int CG = 256 / L, CH = CG * CPT, Np = L * NS, ITEMS = TB * CH / 8, BCN = TB * 2 * Np / 4, BCV = (BCN + 255) / 256;
  constexpr bool AHEAD = NS * CPT <= 4;  // (registers)
  static_assert(ITEMS <= 256 && TB % 4 == 0, "tile");
  __shared__ __attribute__((aligned(16))) float ds[TB][CH];      // dt; then y
  __shared__ __attribute__((aligned(16))) float xs[TB][CH];      // dt u
  __shared__ __attribute__((aligned(16))) float bc[TB][2 * Np];  // B | C
  const int tid = threadIdx.x, ch = tid / L, part = tid % L, c0 = blockIdx.x * CH, b = blockIdx.y;
  const int seg = MODE == SCAN_WHOLE ? 0 : blockIdx.z, t_seg = seg * p.seg_len;
  const int r0 = p.cu[b] + t_seg, left = p.cu[b + 1] - r0;
  const bool last = MODE == SCAN_WHOLE || left <= p.seg_len;
  if (left <= 0 || (MODE == SCAN_SUMMARY && last)) return;
  const int n = last ? left : p.seg_len;
  const int C = p.d.C;
  float S[CPT][NS], A[CPT][NS], total[CPT];
  float* sp[CPT];
  const bool fresh = MODE == SCAN_SUMMARY || (MODE == SCAN_WHOLE && p.pos[r0] == 0);
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const size_t c = min(c0 + ch + i * CG, C - 1);
    sp[i] = p.state + ((size_t)p.slot[b] * C + c) * Np + part * NS;
    float* at = MODE == SCAN_WHOLE ? sp[i] : p.starts + (((size_t)b * p.segs + seg) * C + c) * Np + part * NS;
    if (MODE == SCAN_SUMMARY) sp[i] = at;
    total[i] = 0.f;
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const float v = fresh ? 0.f : at[j];
      S[i][j] = v;
      A[i][j] = p.A[c * Np + part * NS + j];
    }
  }
  // this thread's 8 channels of one token of a tile (CH and C are multiples of 8)
  const int it = tid / (CH / 8), ic = (tid % (CH / 8)) * 8, cc = c0 + ic;
  const bool item = tid < ITEMS && cc < C;
  const int ccl = min(cc, C - 8);
  float nu[8], nd[8], nz[8], bias[8], skip[8];
  f32x4 nb[BCV];
  ElemIO<float>::load8(p.bias + ccl, bias);
  ElemIO<float>::load8(p.skip + ccl, skip);
  auto fetch = [&](int t0) {  // rows past the portion are clamped, and nulled when they are used
    const long row = r0 + min(t0 + min(it, TB - 1), n - 1);
    ElemIO<AT>::load8((const AT*)p.u + row * C + ccl, nu);
    proj8<float>(p.dt, row, ccl, nd);
    proj8<PT>(p.y, row, p.d.z_col + ccl, nz);
#pragma unroll
    for (int k = 0; k < BCV; ++k) {
      const int e = min(k * 256 + tid, BCN - 1) * 4, t = e / (2 * Np), j = e % (2 * Np);
      const int col = j < Np ? p.d.b_col + j : p.d.c_col + j - Np;
      nb[k] = *reinterpret_cast<const f32x4*>((const float*)p.bc.p + (long)(r0 + min(t0 + t, n - 1)) * p.bc.ld + col);
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += TB) {
    float u[8], z[8];
    const bool live = item && t0 + it < n;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      u[j] = nu[j];
      z[j] = nz[j];
    }
    if (item) {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        nd[j] = live ? softplus_f(nd[j] + bias[j]) : 0.f;
        nu[j] = nd[j] * u[j];
      }
      ElemIO<float>::store8(&ds[it][ic], nd);
      ElemIO<float>::store8(&xs[it][ic], nu);
    }
#pragma unroll
    for (int k = 0; k < BCV; ++k)
      if (BCN % 256 == 0 || k * 256 + tid < BCN) *reinterpret_cast<f32x4*>(&bc[0][0] + (k * 256 + tid) * 4) = nb[k];
    __syncthreads();
    if (t0 + TB < n) fetch(t0 + TB);
    // the values of the next four tokens are read under the current ones
    float dn[4][CPT], xn[4][CPT], bn[4][NS], cn[4][NS];
    auto read4 = [&](int t) {
#pragma unroll
      for (int q = 0; q < 4; ++q) {
#pragma unroll
        for (int i = 0; i < CPT; ++i) {
          dn[q][i] = ds[t + q][ch + i * CG];
          xn[q][i] = xs[t + q][ch + i * CG];
        }
#pragma unroll
        for (int j = 0; j < NS; ++j) {
          bn[q][j] = bc[t + q][part * NS + j];
          cn[q][j] = bc[t + q][Np + part * NS + j];
        }
      }
    };
    if (AHEAD) read4(0);
#pragma unroll 1
    for (int t = 0; t < TB; t += 4) {
      if (!AHEAD) read4(t);
      float dv[4][CPT], xv[4][CPT], br[4][NS], cr[4][NS], y[CPT][4];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
#pragma unroll
        for (int i = 0; i < CPT; ++i) {
          dv[q][i] = dn[q][i];
          xv[q][i] = xn[q][i];
        }
#pragma unroll
        for (int j = 0; j < NS; ++j) {
          br[q][j] = bn[q][j];
          cr[q][j] = cn[q][j];
        }
      }
      if (AHEAD) read4(min(t + 4, TB - 4));
#pragma unroll
      for (int q = 0; q < 4; ++q)
#pragma unroll
        for (int i = 0; i < CPT; ++i) {
          y[i][q] = 0.f;
          if (MODE == SCAN_SUMMARY) total[i] += dv[q][i];
#pragma unroll
          for (int j = 0; j < NS; ++j) {
            S[i][j] = fmaf(__builtin_amdgcn_exp2f(dv[q][i] * A[i][j]), S[i][j], xv[q][i] * br[q][j]);
            if (MODE != SCAN_SUMMARY) y[i][q] = fmaf(S[i][j], cr[q][j], y[i][q]);
          }
        }
      if (MODE == SCAN_SUMMARY) continue;
      const bool b0 = part & 1, b1 = part & 2;
#pragma unroll
      for (int i = 0; i < CPT; ++i) {
        const float v0 = (b0 ? y[i][1] : y[i][0]) + quad_xor1(b0 ? y[i][0] : y[i][1]);
        const float v1 = (b0 ? y[i][3] : y[i][2]) + quad_xor1(b0 ? y[i][2] : y[i][3]);
        const float r = across_quads<L>((b1 ? v1 : v0) + quad_xor2(b1 ? v0 : v1));
        if (part < 4) ds[t + part][ch + i * CG] = r;
      }
    }
    __syncthreads();
    if (MODE != SCAN_SUMMARY && live) {
      float o[8];
      ElemIO<float>::load8(&ds[it][ic], o);
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = fmaf(skip[j], u[j], o[j]) * silu_f(z[j]);
      ElemIO<AT>::store8((AT*)p.out + (size_t)(r0 + t0 + it) * C + cc, o);
    }
  }
#pragma unroll
  for (int i = 0; i < CPT; ++i)
    if (c0 + ch + i * CG < C && (last || MODE == SCAN_SUMMARY)) {
#pragma unroll
      for (int j = 0; j < NS; ++j) sp[i][j] = S[i][j];
      if (MODE == SCAN_SUMMARY && part == 0) p.sums[((size_t)b * p.segs + seg) * C + c0 + ch + i * CG] = total[i];
    }
}

// the segments' summaries -> their start states; four state entries a thread
__global__ __launch_bounds__(256) void selective_combine_kernel(SelScan p) {
  const int Np = p.d.Np, C = p.d.C, b = blockIdx.y, e = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int r0 = p.cu[b], n = p.cu[b + 1] - r0;
  if (n <= 0 || e >= C * Np) return;
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  if (p.pos[r0] != 0) S = *reinterpret_cast<const f32x4*>(p.state + (size_t)p.slot[b] * C * Np + e);
  const f32x4 A = *reinterpret_cast<const f32x4*>(p.A + e);
  for (int g = 0; g * p.seg_len < n; ++g) {
    float* at = p.starts + ((size_t)b * p.segs + g) * C * Np + e;
    const bool more = (g + 1) * p.seg_len < n;
    const f32x4 loc = more ? *reinterpret_cast<const f32x4*>(at) : S;
    const float sum = more ? p.sums[((size_t)b * p.segs + g) * C + e / Np] : 0.f;
    *reinterpret_cast<f32x4*>(at) = S;
#pragma unroll
    for (int j = 0; j < 4; ++j) S[j] = fmaf(__builtin_amdgcn_exp2f(sum * A[j]), S[j], loc[j]);
  }
}

// Segments of the longest portion: enough that every SIMD has several waves, none shorter than 256 tokens.  1: not cut.
int selective_segments(SelectiveShape d, int chunks, int max_q) {
  const long waves = (long)chunks * d.C / 16;  // four lanes a channel
  if (waves < 1 || waves >= 2048 || max_q < 512) return 1;
  const long want = (4096 + waves - 1) / waves, most = max_q / 256;
  return (int)(want < most ? want : most);
}

static bool bad_shape(const SelectiveShape& d) {
  return d.C < 8 || d.C % 8 || d.Np != selective_state_width(d.Np) || d.rank < 0 || d.b_col % 4 || d.c_col % 4 || d.z_col % 8;
}

int selective_scan(const void* u, int act_f32, SelectiveShape d, Proj dt, Proj bc, Proj y, const float* A, const float* dt_bias,
                   const float* skip, float* state, const int* slot, const int* pos, const int* cu, int chunks, int max_q,
                   int segs, float* ws, void* out, hipStream_t s) {
  if (chunks <= 0 || max_q <= 0) return 0;
  if (segs < 1 || segs > 65535 || (segs > 1 && !ws)) return hipErrorInvalidValue;
  if (bad_shape(d) || y.S < 1 || y.ld % 8 || y.slab % 8 || !dt.f32 || dt.S != 1 || dt.ld % 4 || !bc.f32 || bc.S != 1 || bc.ld % 4 || chunks > 65535)
    return hipErrorInvalidValue;
  SelScan p{u, d, dt, bc, y, A, dt_bias, skip, state, slot, pos, cu, out, 0, segs, nullptr, nullptr};
  p.seg_len = segs > 1 ? ((max_q + segs - 1) / segs + 63) / 64 * 64 : max_q;
  if (segs > 1) {
    p.starts = ws;
    p.sums = ws + (size_t)chunks * segs * d.C * d.Np;
  }
  // lanes per channel: more of them when the channels alone leave SIMDs without a wave
  const long waves = (long)chunks * d.C / 16 * segs;
#define SEL_M(PT, AT, L, NS, CPT, TB, MODE)                                                                          \
  hipLaunchKernelGGL((selective_scan_kernel<PT, AT, L, NS, CPT, TB, MODE>),                                          \
                     dim3((d.C + 256 / L * CPT - 1) / (256 / L * CPT), chunks, segs), dim3(256), 0, s, p)
#define SEL_L(PT, AT, L, NS, CPT, TB)                                                                                \
  do {                                                                                                               \
    if (segs == 1) {                                                                                                 \
      SEL_M(PT, AT, L, NS, CPT, TB, SCAN_WHOLE);                                                                     \
    } else {                                                                                                         \
      SEL_M(PT, AT, L, NS, CPT, TB, SCAN_SUMMARY);                                                                   \
      hipLaunchKernelGGL(selective_combine_kernel, dim3((d.C * d.Np / 4 + 255) / 256, chunks), dim3(256), 0, s, p);  \
      SEL_M(PT, AT, L, NS, CPT, TB, SCAN_SEGMENT);                                                                   \
    }                                                                                                                \
  } while (0)
#define SEL_N(PT, AT)                                      \
  do {                                                     \
    switch (d.Np) {                                        \
      case 16:                                             \
        if (waves >= 4096) SEL_L(PT, AT, 4, 4, 2, 16);     \
        else if (waves >= 1024) SEL_L(PT, AT, 4, 4, 1, 32); \
        else if (waves >= 256) SEL_L(PT, AT, 8, 2, 1, 64); \
        else SEL_L(PT, AT, 16, 1, 1, 64);                  \
        break;                                             \
      case 32:                                             \
        if (waves >= 1024) SEL_L(PT, AT, 4, 8, 1, 32);     \
        else SEL_L(PT, AT, 16, 2, 1, 64);                  \
        break;                                             \
      case 48: SEL_L(PT, AT, 4, 12, 1, 32); break;         \
      case 64: SEL_L(PT, AT, 8, 8, 1, 32); break;          \
      case 128: SEL_L(PT, AT, 16, 8, 1, 32); break;        \
      case 256: SEL_L(PT, AT, 16, 16, 1, 16); break;       \
      default: return hipErrorInvalidValue;                \
    }                                                      \
  } while (0)
  DAB_PROJ_DISPATCH(y, act_f32, SEL_N);
#undef SEL_N
#undef SEL_L
#undef SEL_M
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------
// one decoded token per sequence

struct SelStep {
  const void* u;        // [*, C]
  SelectiveShape d;
  const void* dt_w;     // [C, rank padded]: bf16 fragments (ops.shuffle_weights) or fp32 rows
  const void* low;      // [*, rank padded] low-rank steps: bf16, or fp32 with bc's row stride
  Proj bc;              // fp32 rows of the narrow projection
  const float* A;
  const float* bias;
  const float* skip;
  float* state;
  const int* slot;
  const int* pos;
  int row0, B;
  void* out;            // [*, C]: the gate on entry
};

// What a wave needs of SW sequences for its 16 channels, requested at once
template <int NS, int SW>
struct StepRegs {
  f32x4 S[SW][NS / 4];
  float u[SW], z[SW];
};

// A wave: 16 channels (4 lanes each, NS state entries a lane).  WIDE: the four waves hold neighbouring channels and walk 16
// sequences, SW at a time, the next ones requested under the current; else they hold the same channels, SW sequences each.
// bf16: W_dt low of a wave's channels and up to 16 sequences is one MFMA tile.
template <typename AT, int NS, int SW, bool WIDE>
__global__ __launch_bounds__(256) void selective_step_kernel(SelStep p) {
  constexpr int Np = 4 * NS, SEQS = WIDE ? 16 : SW;  // sequences of a wave
  __shared__ float dts[4][SEQS][16];
  __shared__ __attribute__((aligned(16))) float bcs[4][SEQS][2 * Np];  // B | C
  const int tid = threadIdx.x, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lane = tid & 63, g = lane >> 4, li = lane & 15, part = lane & 3;
  const int blk = WIDE ? blockIdx.x * 4 + w : blockIdx.x, c = blk * 16 + (lane >> 2);
  const int C = p.d.C, R = p.d.rank, sw0 = blockIdx.y * (WIDE ? 16 : 4 * SW), s0 = WIDE ? sw0 : sw0 + w * SW;
  if (s0 >= p.B || blk * 16 >= C) return;  // the whole wave (no barrier follows)
  // slots and positions of the wave's sequences, a lane each (read back as scalars); sequences past the last are the last
  const int mine = min(s0 + min(li, SEQS - 1), p.B - 1), slots = p.slot[mine], places = p.pos[p.row0 + mine];
  const int cell = c * Np + part * NS;  // of a slot's state
  auto state = [&](int s) { return p.state + (size_t)__builtin_amdgcn_readlane(slots, s) * C * Np + cell; };
  auto request = [&](int at, StepRegs<NS, SW>& q) {
#pragma unroll
    for (int s = 0; s < SW; ++s) {
      const float* sp = state(at + s);
      const size_t cell = (size_t)(p.row0 + min(s0 + at + s, p.B - 1)) * C + c;
#pragma unroll
      for (int j = 0; j < NS / 4; ++j) q.S[s][j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(sp + 4 * j));
      q.u[s] = ElemIO<AT>::load((const AT*)p.u + cell);
      q.z[s] = ElemIO<AT>::load((const AT*)p.out + cell);
    }
  };
  StepRegs<NS, SW> q;
  request(0, q);
  for (int i = lane * 4; i < SEQS * 2 * Np; i += 256) {
    const int s = i / (2 * Np), j = i % (2 * Np);
    const float* br = (const float*)p.bc.p + (size_t)(p.row0 + min(s0 + s, p.B - 1)) * p.bc.ld;
    *reinterpret_cast<f32x4*>(&bcs[w][0][0] + i) = *reinterpret_cast<const f32x4*>(br + (j < Np ? p.d.b_col + j : p.d.c_col + j - Np));
  }
  f32x4 A[NS / 4];
#pragma unroll
  for (int j = 0; j < NS / 4; ++j) A[j] = *reinterpret_cast<const f32x4*>(p.A + (size_t)c * Np + part * NS + 4 * j);
  const float bias = p.bias[c], skip = p.skip[c];
  if constexpr (sizeof(AT) == 2) {
    const bf16* wp = (const bf16*)p.dt_w + (size_t)blk * (R / 32) * 512 + lane * 8;
    const bf16* lp = (const bf16*)p.low + (size_t)(p.row0 + min(sw0 + li, p.B - 1)) * R + 8 * g;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 0; k < R / 32; ++k)
      acc = mfma16(*reinterpret_cast<const bf16x8*>(wp + (size_t)k * 512), *reinterpret_cast<const bf16x8*>(lp + 32 * k), acc);
    if (WIDE || li / SW == w) {  // channel 4 g + r of sequence sw0 + li
#pragma unroll
      for (int r = 0; r < 4; ++r) dts[w][li % SEQS][4 * g + r] = acc[r];
    }
  } else {
#pragma unroll 1
    for (int s = 0; s < SEQS && s0 + s < p.B; ++s) {
      const float* wp = (const float*)p.dt_w + (size_t)c * R;
      const float* lp = (const float*)p.low + (size_t)(p.row0 + s0 + s) * p.bc.ld;
      float a = 0.f;
      for (int k = part * 4; k < R; k += 16)
#pragma unroll
        for (int e = 0; e < 4; ++e) a = fmaf(wp[k + e], lp[k + e], a);
      a += quad_xor1(a);
      a += quad_xor2(a);
      if (part == 0) dts[w][s][lane >> 2] = a;
    }
  }
  // (a wave reads what it wrote itself)
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll 1
  for (int at = 0; at < SEQS; at += SW) {
    if (s0 + at >= p.B) break;
    StepRegs<NS, SW> cur = q;
    if (at + SW < SEQS) request(at + SW, q);
#pragma unroll
    for (int s = 0; s < SW; ++s) {
      const float dt = softplus_f(dts[w][at + s][lane >> 2] + bias), x = dt * cur.u[s];
      const float* bc = &bcs[w][at + s][part * NS];
      const bool fresh = __builtin_amdgcn_readlane(places, at + s) == 0, live = s0 + at + s < p.B;
      float* sp = state(at + s);
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < NS / 4; ++j) {
        const f32x4 bv = *reinterpret_cast<const f32x4*>(bc + 4 * j), cv = *reinterpret_cast<const f32x4*>(bc + Np + 4 * j);
        f32x4 nv;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float prev = fresh ? 0.f : cur.S[s][j][e];
          nv[e] = fmaf(__builtin_amdgcn_exp2f(dt * A[j][e]), prev, x * bv[e]);
          y = fmaf(nv[e], cv[e], y);
        }
        if (live) __builtin_nontemporal_store(nv, reinterpret_cast<f32x4*>(sp + 4 * j));
      }
      y += quad_xor1(y);
      y += quad_xor2(y);
      if (live && part == 0)
        ElemIO<AT>::store((AT*)p.out + (size_t)(p.row0 + s0 + at + s) * C + c, fmaf(skip, cur.u[s], y) * silu_f(cur.z[s]));
    }
  }
}

int selective_step(const void* u, int act_f32, SelectiveShape d, const void* dt_w, const void* low, Proj bc, const float* A,
                   const float* dt_bias, const float* skip, float* state, const int* slot, const int* pos,
                   int row0, int B, void* out, hipStream_t s) {
  if (B <= 0) return 0;
  if (bad_shape(d) || d.C % 16 || d.rank < 32 || d.rank % 32 || !bc.f32 || bc.S != 1 || bc.ld % 4 || B > 65535)
    return hipErrorInvalidValue;
  SelStep p{u, d, dt_w, low, bc, A, dt_bias, skip, state, slot, pos, row0, B, out};
  const bool wide = B > 16 && d.C % 64 == 0;
#define STEP_L(AT, NS, SW, WIDE)                                                                                   \
  hipLaunchKernelGGL((selective_step_kernel<AT, NS, SW, WIDE>),                                                    \
                     WIDE ? dim3((d.C + 63) / 64, (B + 15) / 16) : dim3(d.C / 16, (B + 4 * SW - 1) / (4 * SW)), dim3(256), 0, s, p)
#define STEP_N(AT)                              \
  do {                                              \
    switch (d.Np) {                                 \
      case 16:                                      \
        if (wide) STEP_L(AT, 4, 4, true);       \
        else STEP_L(AT, 4, 1, false);           \
        break;                                      \
      case 32:                                      \
        if (wide) STEP_L(AT, 8, 2, true);       \
        else STEP_L(AT, 8, 1, false);           \
        break;                                      \
      case 48: STEP_L(AT, 12, 1, false); break; \
      case 64: STEP_L(AT, 16, 1, false); break; \
      case 128: STEP_L(AT, 32, 1, false); break; \
      case 256: STEP_L(AT, 64, 1, false); break; \
      default: return hipErrorInvalidValue;         \
    }                                               \
  } while (0)
  if (act_f32) STEP_N(float);
  else STEP_N(bf16);
#undef STEP_N
#undef STEP_L
  return hipGetLastError();
}

}  // namespace dab
