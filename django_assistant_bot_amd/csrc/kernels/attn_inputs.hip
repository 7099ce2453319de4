// The step between a layer's input projection and its attention: columns [q heads | k heads | v heads] of D each ->
//   bias, short causal convolution over time per channel, RMS norm of q and k with gains (each head, or all heads of q and of
//   k at once), rotation of neighbouring pairs, query temperature, mix of the values with another layer's; q rows out, k / v
//   into the paged cache.
//
// Past inputs of the convolution live in a ring of ``taps`` entries per slot, entry p % taps holding the input of position p
// (recurrent.hip has the same); entries before position 0 are never read.  A decoded token reads its past from the ring and
// writes its own entry, which nothing in its step reads; a prompt portion is followed by attn_ring, which writes the last
// ``taps`` inputs.
#include <type_traits>

#include "launchers.h"
#include "proj.h"

namespace dab {

// the sum over groups of LPH neighbouring lanes (8 .. 64), in every lane
template <int LPH>
__device__ __forceinline__ float sum_lanes(float v) {
  const auto dpp = [](float x, auto ctrl) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), decltype(ctrl)::value, 0xf, 0xf, true));
  };
  v += dpp(v, std::integral_constant<int, 0xb1>{});   // neighbours
  v += dpp(v, std::integral_constant<int, 0x4e>{});   // pairs
  v += dpp(v, std::integral_constant<int, 0x141>{});  // quads, mirrored within 8
  if (LPH >= 16) v += dpp(v, std::integral_constant<int, 0x140>{});  // eights, mirrored within 16
#pragma unroll
  for (int o = 16; o < LPH; o <<= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// 8 elements as they are stored
template <typename T>
struct Raw8 {
  u32x4 v[sizeof(T) / 2];
  __device__ __forceinline__ void load(const T* p) {
#pragma unroll
    for (int i = 0; i < (int)sizeof(T) / 2; ++i) v[i] = reinterpret_cast<const u32x4*>(p)[i];
  }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < (int)sizeof(T) / 2; ++i) v[i] = u32x4{0, 0, 0, 0};
  }
  __device__ __forceinline__ void get(float (&f)[8]) const {
    if constexpr (sizeof(T) == 2) {
      unpack8(v[0], f);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = __uint_as_float(v[j / 4][j % 4]);
    }
  }
};

// What a workgroup's tokens share, in LDS: cosines and sines (1, 0 behind the rotated pairs), query temperatures, cache rows
// of key head 0 (-1: none)
template <int NT, int PAIRS>
struct TokenTables {
  __attribute__((aligned(16))) float2 cs[NT * PAIRS];
  float temp[NT];
  int row[NT];

  __device__ __forceinline__ void fill(const AttnInputs& p, int r0, int pos0, int nt) {  // tokens in rows r0 .., from position pos0
    if (p.rot) {
      for (int e = threadIdx.x; e < nt * PAIRS; e += blockDim.x) {
        const int t = e / PAIRS, pr = e % PAIRS;
        float c = 1.f, s = 0.f;
        if (2 * pr < p.rot) {
          const double turns = (double)(pos0 + t) * p.turns[pr];
          sincos_turn(turns - rint(turns), s, c);
          c *= p.rot_mul;
          s *= p.rot_mul;
        }
        cs[e] = make_float2(c, s);
      }
    }
    const int t = threadIdx.x;
    if (t < nt) {
      temp[t] = p.t_coef == 0.f ? 1.f : 1.f + p.t_coef * logf((float)((pos0 + t + 1) / p.t_every) + 1.f);
      const int64_t slot = p.slots[r0 + t];
      const unsigned u = (unsigned)slot;
      row[t] = slot < 0 ? -1 : (int)(u / (unsigned)p.bs * (p.G * p.bs) + u % (unsigned)p.bs);
    }
  }
};

// q and k: x *= r * gain, the rotation, and for q the temperature (already in r); then rows and cache.  v: the mix, then the cache
template <typename AT, int NT, int PAIRS>
__device__ __forceinline__ void put_head(const AttnInputs& p, const TokenTables<NT, PAIRS>& tab, int r0, int t, int hd, int col,
                                         float r, const float (&gain)[8], float (&x)[8]) {
  AT* dst;
  if (hd < p.H + p.G) {
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= r * gain[j];
    if (p.rot) {
      const f32x4* w = reinterpret_cast<const f32x4*>(&tab.cs[t * PAIRS + col / 2]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float c = w[e / 2][2 * (e % 2)], s = w[e / 2][2 * (e % 2) + 1], u = x[2 * e], v = x[2 * e + 1];
        x[2 * e] = u * c - v * s;
        x[2 * e + 1] = v * c + u * s;
      }
    }
    if (hd < p.H) {
      dst = (AT*)p.q + ((size_t)(r0 + t) * p.H + hd) * p.D;
    } else {
      if (tab.row[t] < 0) return;
      dst = (AT*)p.kc + (size_t)(unsigned)(tab.row[t] + (hd - p.H) * p.bs) * p.D;
    }
  } else {
    const int g = hd - p.H - p.G;
    if (p.mix && col < p.first_w) {
      AT* q = (AT*)p.first + ((size_t)(r0 + t) * p.G + g) * p.first_w + col;
      if (p.mix == 1) {
        ElemIO<AT>::store8(q, x);
      } else {
        float v[8];
        ElemIO<AT>::load8(q, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = fmaf(p.lam, v[j] - x[j], x[j]);
      }
    }
    if (tab.row[t] < 0) return;
    dst = (AT*)p.vc + (size_t)(unsigned)(tab.row[t] + g * p.bs) * p.D;
  }
  ElemIO<AT>::store8(dst + col, x);
}

// Prompt portions, finished projections, a norm per head, at most four taps: a workgroup takes 8 tokens, groups of LPH lanes
// walk heads.  All of a head's rows are requested together; a lane convolves its 8 columns along them.
template <typename AT, int LPH, bool CONV>
__global__ __launch_bounds__(256) void attn_span_kernel(AttnInputs p) {
  constexpr int NT = 8, PAIRS = 4 * LPH, PAST = CONV ? 3 : 0;
  __shared__ TokenTables<NT, PAIRS> tab;
  const int grp = threadIdx.x / LPH, ng = 256 / LPH, col = threadIdx.x % LPH * 8;
  const int heads = p.H + 2 * p.G, C = heads * p.D;
  const int r0 = p.cu[blockIdx.y], n = p.cu[blockIdx.y + 1] - r0, t0 = blockIdx.x * NT;
  if (t0 >= n) return;
  const int nt = min(NT, n - t0), pos0 = p.positions[r0];
  tab.fill(p, r0 + t0, pos0 + t0, nt);
  __syncthreads();
  const AT* y = (const AT*)p.y.p + (size_t)(r0 + t0) * p.y.ld + p.col0;
  const AT* ring = CONV ? (const AT*)p.ring + (size_t)p.slot[blockIdx.y] * p.taps * C : nullptr;
  for (int h0 = blockIdx.z * ng; h0 < heads; h0 += ng * gridDim.z) {  // (uniform: the groups of a wave reduce together)
    const int hd = min(h0 + grp, heads - 1), at = hd * p.D + col;
    const bool on = h0 + grp < heads && col < p.D;
    const int ld_at = min(at, C - 8);  // (columns behind a head's end are not used)
    Raw8<AT> raw[NT + PAST];
#pragma unroll
    for (int i = 0; i < NT; ++i) raw[PAST + i].load(y + (size_t)min(i, nt - 1) * p.y.ld + ld_at);
    float bias[8], w[4][8], gain[8];
    ElemIO<float>::load8(p.gain + min(ld_at, (p.H + p.G) * p.D - 8), gain);
#pragma unroll
    for (int j = 0; j < 8; ++j) bias[j] = 0.f;
    if (p.bias) ElemIO<float>::load8(p.bias + ld_at, bias);
    if constexpr (CONV) {
#pragma unroll
      for (int k = 0; k < 3; ++k) {  // raw[k]: the input 3 - k tokens before t0
        if (t0 > 0) raw[k].load(y - (size_t)(3 - k) * p.y.ld + ld_at);
        else if (3 - k < p.taps && pos0 >= 3 - k) raw[k].load(ring + (size_t)((pos0 - 3 + k) % p.taps) * C + ld_at);
        else raw[k].zero();
      }
#pragma unroll
      for (int k = 0; k < 4; ++k) {  // w[k] meets the input 3 - k tokens back
        ElemIO<float>::load8(p.conv + (size_t)max(k - 4 + p.taps, 0) * C + ld_at, w[k]);
        if (k < 4 - p.taps) {
#pragma unroll
          for (int j = 0; j < 8; ++j) w[k][j] = 0.f;
        }
      }
    }
    float win[4][8];
    if constexpr (CONV) {
#pragma unroll
      for (int k = 0; k < 3; ++k) {
        raw[k].get(win[k]);
        if (t0 > 0) {  // (the ring's entries have their bias)
#pragma unroll
          for (int j = 0; j < 8; ++j) win[k][j] += bias[j];
        }
      }
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      float x[8];
      raw[PAST + t].get(x);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] += bias[j];
      if constexpr (CONV) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          win[(t + 3) % 4][j] = x[j];
          x[j] *= w[3][j];
#pragma unroll
          for (int k = 0; k < 3; ++k) x[j] = fmaf(w[k][j], win[(t + k) % 4][j], x[j]);
        }
      }
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
      if (col >= p.D) ss = 0.f;
      ss = sum_lanes<LPH>(ss);
      const float r = __builtin_amdgcn_rsqf(fmaf(ss, p.inv_q, p.eps)) * (hd < p.H ? tab.temp[t] : 1.f);
      if (on && t < nt) put_head<AT>(p, tab, r0 + t0, t, hd, col, r, gain, x);
    }
  }
}

// Prompt portions, finished projections, no convolution, one norm over all q and one over all k heads: a workgroup takes a
// token, a group of LPH lanes holds up to HR heads of it.
template <typename AT, int LPH, int HR>
__global__ __launch_bounds__(256) void attn_whole_kernel(AttnInputs p) {
  constexpr int PAIRS = 4 * LPH;
  __shared__ TokenTables<1, PAIRS> tab;
  __shared__ float red[2][4];
  const int grp = threadIdx.x / LPH, ng = 256 / LPH, col = threadIdx.x % LPH * 8;
  const int heads = p.H + 2 * p.G, C = heads * p.D;
  const int r0 = p.cu[blockIdx.y], t = blockIdx.x;
  if (t >= p.cu[blockIdx.y + 1] - r0) return;
  const AT* y = (const AT*)p.y.p + (size_t)(r0 + t) * p.y.ld + p.col0;
  Raw8<AT> raw[HR];
#pragma unroll
  for (int i = 0; i < HR; ++i) raw[i].load(y + min((grp + i * ng) * p.D + col, C - 8));
  float x[HR][8], sq = 0.f, sk = 0.f;
  tab.fill(p, r0 + t, p.positions[r0] + t, 1);
#pragma unroll
  for (int i = 0; i < HR; ++i) {
    const int hd = grp + i * ng;
    raw[i].get(x[i]);
    if (p.bias) {
      float b[8];
      ElemIO<float>::load8(p.bias + min(hd * p.D + col, C - 8), b);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += b[j];
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(x[i][j], x[i][j], ss);
    if (col < p.D) {
      sq += hd < p.H ? ss : 0.f;
      sk += hd >= p.H && hd < p.H + p.G ? ss : 0.f;
    }
  }
  sq = sum_lanes<64>(sq);
  sk = sum_lanes<64>(sk);
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = sq;
    red[1][threadIdx.x >> 6] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  const float rq = __builtin_amdgcn_rsqf(fmaf(sq, p.inv_q, p.eps)) * tab.temp[0], rk = __builtin_amdgcn_rsqf(fmaf(sk, p.inv_k, p.eps));
  if (col >= p.D) return;
#pragma unroll
  for (int i = 0; i < HR; ++i) {
    const int hd = grp + i * ng;
    if (hd >= heads) break;
    float gain[8];
    ElemIO<float>::load8(p.gain + min(hd, p.H + p.G - 1) * p.D + col, gain);
    put_head<AT>(p, tab, r0 + t, 0, hd, col, hd < p.H ? rq : rk, gain, x[i]);
  }
}

// Everything else: decoded tokens, split-K slabs, many taps, wide heads.  A workgroup takes NT tokens of one portion (CU) or one
// decoded token; groups of LPH lanes walk heads, a lane owning columns 8 (lane + LPH i) .. + 7, i < NP, of a head.  Past inputs
// are fetched for every token.  WHOLE: the norm runs over all heads, so the workgroup first sums squares (NT is 1).
template <typename PT, typename AT, int LPH, int NP, int NT, bool WHOLE, bool CU>
__global__ __launch_bounds__(CU ? 256 : 1024) void attn_inputs_kernel(AttnInputs p) {
  constexpr int PAIRS = 4 * LPH * NP;
  static_assert(!WHOLE || NT == 1, "the norm over all heads takes a token at a time");
  __shared__ TokenTables<NT, PAIRS> tab;
  __shared__ float red[2][16];
  const int grp = threadIdx.x / LPH, lane = threadIdx.x % LPH, ng = blockDim.x / LPH;
  const int heads = p.H + 2 * p.G, C = heads * p.D;
  int r0, n, t0 = 0;  // first row of the portion, its tokens, the first one taken here
  if (CU) {
    r0 = p.cu[blockIdx.y];
    n = p.cu[blockIdx.y + 1] - r0;
    t0 = blockIdx.x * NT;
    if (t0 >= n) return;
  } else {
    r0 = p.row0 + blockIdx.x;
    n = 1;
  }
  const int nt = min(NT, n - t0), pos0 = p.positions[r0];
  AT* ring = (AT*)p.ring + (p.conv ? (size_t)p.slot[CU ? blockIdx.y : blockIdx.x] * p.taps * C : 0);
  tab.fill(p, r0 + t0, pos0 + t0, nt);
  int col[NP];
  bool in[NP];
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int d = 8 * (lane + LPH * i);
    in[i] = d < p.D;
    col[i] = min(d, p.D - 8);
  }
  // the convolved value of token t of the portion at the lane's columns of head hd
  auto value = [&](int t, int hd, int i, float(&x)[8]) {
    const int at = hd * p.D + col[i];
    float b[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) b[j] = 0.f;
    if (p.bias) ElemIO<float>::load8(p.bias + at, b);
    proj8<PT>(p.y, r0 + t, p.col0 + at, x);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] += b[j];
    if (!p.conv) return;
    const float* wp = p.conv + at;
    AT* mine = ring + at;
    if (!CU && in[i]) ElemIO<AT>::store8(mine + (size_t)(pos0 % p.taps) * C, x);  // (read by no token of this step)
    float w[8];
    ElemIO<float>::load8(wp + (size_t)(p.taps - 1) * C, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= w[j];
    if (CU) {
      for (int k = 1; k < p.taps && k <= pos0 + t; ++k) {  // inputs of the portion, then of the ring
        float u[8];
        if (k <= t) {
          proj8<PT>(p.y, r0 + t - k, p.col0 + at, u);
#pragma unroll
          for (int j = 0; j < 8; ++j) u[j] += b[j];
        } else {
          ElemIO<AT>::load8(mine + (size_t)((pos0 + t - k) % p.taps) * C, u);
        }
        ElemIO<float>::load8(wp + (size_t)(p.taps - 1 - k) * C, w);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = fmaf(w[j], u[j], x[j]);
      }
      return;
    }
    const int now = pos0 % p.taps;
    for (int k0 = 1; k0 < p.taps; k0 += 4) {  // four past inputs requested at a time
      float u[4][8], tap[4][8];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int k = min(k0 + q, p.taps - 1), e = now >= k ? now - k : now - k + p.taps;
        ElemIO<AT>::load8(mine + (size_t)e * C, u[q]);
        ElemIO<float>::load8(wp + (size_t)(p.taps - 1 - k) * C, tap[q]);
      }
#pragma unroll
      for (int q = 0; q < 4; ++q)
        if (k0 + q < p.taps && k0 + q <= pos0) {
#pragma unroll
          for (int j = 0; j < 8; ++j) x[j] = fmaf(tap[q][j], u[q][j], x[j]);
        }
    }
  };
  float rq = 0.f, rk = 0.f;
  if (WHOLE) {
    float sq = 0.f, sk = 0.f;
    for (int hd = grp; hd < p.H + p.G; hd += ng) {
      float x[8], ss = 0.f;
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        value(t0, hd, i, x);
        if (in[i]) {
#pragma unroll
          for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
        }
      }
      if (hd < p.H) sq += ss;
      else sk += ss;
    }
    sq = sum_lanes<64>(sq);
    sk = sum_lanes<64>(sk);
    if ((threadIdx.x & 63) == 0) {
      red[0][threadIdx.x >> 6] = sq;
      red[1][threadIdx.x >> 6] = sk;
    }
    __syncthreads();
    sq = sk = 0.f;
    for (int i = 0; i < (int)(blockDim.x >> 6); ++i) {
      sq += red[0][i];
      sk += red[1][i];
    }
    rq = __builtin_amdgcn_rsqf(fmaf(sq, p.inv_q, p.eps)) * tab.temp[0];
    rk = __builtin_amdgcn_rsqf(fmaf(sk, p.inv_k, p.eps));
  } else {
    __syncthreads();
  }
  // (uniform trip count: the groups of a wave reduce together)
  for (int h0 = blockIdx.z * ng; h0 < heads; h0 += ng * gridDim.z) {
    const int hd = min(h0 + grp, heads - 1);
    float gain[NP][8];
#pragma unroll
    for (int i = 0; i < NP; ++i) ElemIO<float>::load8(p.gain + min(hd, p.H + p.G - 1) * p.D + col[i], gain[i]);
    for (int t = 0; t < nt; ++t) {
      float x[NP][8], r = hd < p.H ? rq : rk;
#pragma unroll
      for (int i = 0; i < NP; ++i) value(t0 + t, hd, i, x[i]);
      if (!WHOLE) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NP; ++i)
          if (in[i]) {
#pragma unroll
            for (int j = 0; j < 8; ++j) ss = fmaf(x[i][j], x[i][j], ss);
          }
        r = __builtin_amdgcn_rsqf(fmaf(sum_lanes<LPH>(ss), p.inv_q, p.eps)) * (hd < p.H ? tab.temp[t] : 1.f);
      }
#pragma unroll
      for (int i = 0; i < NP; ++i)
        if (in[i] && h0 + grp < heads) put_head<AT>(p, tab, r0 + t0, t, hd, col[i], r, gain[i], x[i]);
    }
  }
}

// the last ``taps`` inputs of every portion into its ring, 8 channels a thread
template <typename PT, typename AT>
__global__ __launch_bounds__(256) void attn_ring_kernel(AttnInputs p) {
  const int C = (p.H + 2 * p.G) * p.D, b = blockIdx.z, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  const int r0 = p.cu[b], n = p.cu[b + 1] - r0, t = n - 1 - (int)blockIdx.y;
  if (t < 0 || c >= C) return;
  float v[8];
  proj8<PT>(p.y, r0 + t, p.col0 + c, v);
  if (p.bias) {
    float w[8];
    ElemIO<float>::load8(p.bias + c, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] += w[j];
  }
  ElemIO<AT>::store8((AT*)p.ring + ((size_t)p.slot[b] * p.taps + (p.positions[r0] + t) % p.taps) * C + c, v);
}

int attn_inputs(AttnInputs p, int act_f32, int rows, int max_q, hipStream_t s) {
  if (rows <= 0) return 0;  // portions (cu) or decoded tokens
  if (p.H < 1 || p.G < 1 || p.D < 8 || p.D % 8 || p.D > 1024 || p.col0 % 8 || p.y.ld % 8 || p.y.slab % 8 || p.y.S < 1 ||
      p.rot < 0 || p.rot % 2 || p.rot > p.D || (p.rot && !p.turns) || p.bs < 1 || p.taps < 1 || p.taps > 16 || !p.gain ||
      (p.taps > 1 && !p.conv) || (p.conv && (!p.ring || !p.slot)) || p.t_every < 1 || (p.mix && (!p.first || p.first_w % 8)) ||
      (p.cu && (max_q < 1 || max_q > (1 << 19) || rows > 65535)))
    return hipErrorInvalidValue;
  const int heads = p.H + 2 * p.G, C = heads * p.D;
  const int lph = p.D <= 64 ? 8 : p.D <= 128 ? 16 : p.D <= 256 ? 32 : 64;
  const bool done = p.cu && p.y.S == 1 && p.y.f32 == act_f32 && p.D <= 256;  // finished rows of prompts
  const bool span = done && !p.whole && (!p.conv || p.taps <= 4);
  const bool held = done && p.whole && !p.conv && heads <= 4 * (256 / lph);
  const int nt = p.cu && !p.whole ? 8 : 1;
  int bt = 256, slices = 1;
  if (p.cu) {
    if (span && (long)rows * ((max_q + 7) / 8) < 1024) slices = (heads * lph + 255) / 256;
  } else {
    bt = (heads * lph + 63) / 64 * 64;
    if (!p.whole && rows < 128 && bt > 256) {  // few decoded tokens: a token's heads over several workgroups
      slices = (bt + 255) / 256;
      bt = 256;
    }
    bt = bt > 1024 ? 1024 : bt;
  }
  const dim3 grid(p.cu ? (max_q + nt - 1) / nt : rows, p.cu ? rows : 1, slices);
#define AI_FAST(AT, LPH)                                                                                       \
  do {                                                                                                         \
    if (held) hipLaunchKernelGGL((attn_whole_kernel<AT, LPH, 4>), grid, dim3(256), 0, s, p);                   \
    else if (p.conv) hipLaunchKernelGGL((attn_span_kernel<AT, LPH, true>), grid, dim3(256), 0, s, p);          \
    else hipLaunchKernelGGL((attn_span_kernel<AT, LPH, false>), grid, dim3(256), 0, s, p);                     \
  } while (0)
#define AI_DONE(AT)                       \
  do {                                    \
    if (lph == 8) AI_FAST(AT, 8);         \
    else if (lph == 16) AI_FAST(AT, 16);  \
    else AI_FAST(AT, 32);                 \
  } while (0)
#define AI_L(PT, AT, LPH, NP, NT, W, CU) \
  hipLaunchKernelGGL((attn_inputs_kernel<PT, AT, LPH, NP, NT, W, CU>), grid, dim3(bt), 0, s, p)
#define AI_K(PT, AT, LPH, NP)                                      \
  do {                                                             \
    if (p.cu && p.whole) AI_L(PT, AT, LPH, NP, 1, true, true);     \
    else if (p.cu) AI_L(PT, AT, LPH, NP, 8, false, true);          \
    else if (p.whole) AI_L(PT, AT, LPH, NP, 1, true, false);       \
    else AI_L(PT, AT, LPH, NP, 1, false, false);                   \
  } while (0)
#define AI_D(PT, AT)                                                                                                \
  do {                                                                                                              \
    if (span || held) AI_DONE(AT);                                                                                  \
    else if (lph == 8) AI_K(PT, AT, 8, 1);                                                                          \
    else if (lph == 16) AI_K(PT, AT, 16, 1);                                                                        \
    else if (lph == 32) AI_K(PT, AT, 32, 1);                                                                        \
    else AI_K(PT, AT, 64, 2);                                                                                       \
    if (p.cu && p.conv)                                                                                             \
      hipLaunchKernelGGL((attn_ring_kernel<PT, AT>), dim3((C / 8 + 255) / 256, p.taps, rows), dim3(256), 0, s, p);  \
  } while (0)
  DAB_PROJ_DISPATCH(p.y, act_f32, AI_D);
#undef AI_D
#undef AI_K
#undef AI_L
#undef AI_DONE
#undef AI_FAST
  return hipGetLastError();
}

}  // namespace dab
