// The step between a layer's input projection and its attention: columns [q heads | k heads | v heads] of D each ->
//   bias, short causal convolution over time per channel, RMS norm of q and k with gains (each head, or all heads of q and of
//   k at once), rotation of neighbouring pairs, query temperature, mix of the values with another layer's; q rows out, k / v
//   into the paged cache.
//
// Past inputs of the convolution live in a ring of ``taps`` entries per slot, entry p % taps holding the input of position p
// (recurrent.hip has the same); entries before position 0 are never read.  A decoded token reads its past from the ring and
// writes its own entry, which nothing in its step reads; a prompt portion is followed by attn_ring, which writes the last
// ``taps`` inputs.
#include "launchers.h"
#include "proj.h"

namespace dab {

__device__ __forceinline__ float sum_lanes(float v, int lph) {
  for (int o = lph / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// A workgroup takes NT tokens of one portion (CU) or one decoded token; groups of LPH lanes walk heads, a lane owning columns
// 8 (lane + LPH i) .. + 7, i < NP, of a head.  K 4: up to four taps, the window of past inputs in registers while a group
// walks its tokens; 0: any number (or no convolution), past inputs fetched for every token.  WHOLE: the norm runs over all heads, so
// the workgroup first sums squares (NT is 1).
template <typename PT, typename AT, int LPH, int NP, int K, int NT, bool WHOLE, bool CU>
__global__ __launch_bounds__(CU ? 256 : 1024) void attn_inputs_kernel(AttnInputs p) {
  constexpr int PAIRS = 4 * LPH * NP;
  static_assert(!WHOLE || NT == 1, "the norm over all heads takes a token at a time");
  static_assert(K != 4 || (NT % 4 == 0 && NP == 1), "whole turns of the window");
  __shared__ __attribute__((aligned(16))) float2 cs[NT * PAIRS];
  __shared__ float temp[NT];
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
  for (int e = threadIdx.x; e < nt * (p.rot / 2); e += blockDim.x) {
    const int t = e / (p.rot / 2), pr = e % (p.rot / 2);
    const double turns = (double)(pos0 + t0 + t) * p.turns[pr];
    float c, s;
    sincos_turn(turns - rint(turns), s, c);
    cs[t * PAIRS + pr] = make_float2(c * p.rot_mul, s * p.rot_mul);
  }
  if ((int)threadIdx.x < nt)
    temp[threadIdx.x] = p.t_coef == 0.f ? 1.f : 1.f + p.t_coef * logf((float)((pos0 + t0 + (int)threadIdx.x + 1) / p.t_every) + 1.f);
  __syncthreads();

  int col[NP];
  bool in[NP];
  // input of token t of the portion (t >= 0) at the lane's columns of head hd, with its bias, as the ring holds it
  auto input = [&](int t, int hd, int i, const float(&b)[8], float(&v)[8]) {
    proj8<PT>(p.y, r0 + t, p.col0 + hd * p.D + col[i], v);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = ElemIO<AT>::round(v[j] + b[j]);
  };
  // input k tokens before token t: of the portion, of the ring, or zero before the sequence
  auto past = [&](int t, int k, int hd, int i, const float(&b)[8], float(&v)[8]) {
    if (t - k >= 0) {
      input(t - k, hd, i, b, v);
    } else if (pos0 + t - k >= 0) {
      ElemIO<AT>::load8(ring + (size_t)((pos0 + t - k) % p.taps) * C + hd * p.D + col[i], v);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = 0.f;
    }
  };
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int d = 8 * (lane + LPH * i);
    in[i] = d < p.D;
    col[i] = min(d, p.D - 8);
  }
  auto bias_of = [&](int hd, int i, float(&b)[8]) {
#pragma unroll
    for (int j = 0; j < 8; ++j) b[j] = 0.f;
    if (p.bias) ElemIO<float>::load8(p.bias + hd * p.D + col[i], b);
  };
  // the convolved value of token t (K = 0)
  auto value = [&](int t, int hd, int i, float(&x)[8]) {
    float b[8];
    bias_of(hd, i, b);
    input(t, hd, i, b, x);
    if (!p.conv) return;
    const float* wp = p.conv + hd * p.D + col[i];
    AT* mine = ring + hd * p.D + col[i];
    if (!CU && in[i]) ElemIO<AT>::store8(mine + (size_t)(pos0 % p.taps) * C, x);  // (read by no token of this step)
    float w[8];
    ElemIO<float>::load8(wp + (size_t)(p.taps - 1) * C, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= w[j];
    if (CU) {
      for (int k = 1; k < p.taps; ++k) {
        float u[8];
        past(t, k, hd, i, b, u);
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
  float rq = 0.f, rk = 0.f;  // WHOLE
  // everything behind the convolution for token t of head hd
  auto finish = [&](int t, int hd, bool on, float(&x)[NP][8], const float(&gain)[NP][8]) {
    const bool is_v = hd >= p.H + p.G;
    const int row = r0 + t;
    float r = WHOLE ? (hd < p.H ? rq : rk) : 0.f;
    if (!WHOLE) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NP; ++i)
        if (in[i]) {
#pragma unroll
          for (int j = 0; j < 8; ++j) ss = fmaf(x[i][j], x[i][j], ss);
        }
      ss = sum_lanes(ss, LPH);
      r = 1.f / sqrtf(ss * p.inv_q + p.eps);
    }
    if (!on) return;
    const int64_t slot = hd < p.H ? 0 : p.slots[row];
    if (!is_v) {
      const float tm = hd < p.H ? temp[t - t0] : 1.f;
#pragma unroll
      for (int i = 0; i < NP; ++i) {
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] *= r * gain[i][j];
        if (col[i] < p.rot) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            if (col[i] + 2 * e >= p.rot) break;
            const float2 w = cs[(t - t0) * PAIRS + col[i] / 2 + e];
            const float u = x[i][2 * e], v = x[i][2 * e + 1];
            x[i][2 * e] = u * w.x - v * w.y;
            x[i][2 * e + 1] = v * w.x + u * w.y;
          }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] *= tm;
      }
    } else if (p.mix) {
      const int g = hd - p.H - p.G;
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        if (!in[i] || col[i] >= p.first_w) continue;
        AT* q = (AT*)p.first + ((size_t)row * p.G + g) * p.first_w + col[i];
        if (p.mix == 1) {
          ElemIO<AT>::store8(q, x[i]);
        } else {
          float v[8];
          ElemIO<AT>::load8(q, v);
#pragma unroll
          for (int j = 0; j < 8; ++j) x[i][j] = fmaf(p.lam, v[j] - x[i][j], x[i][j]);
        }
      }
    }
    if (slot < 0) return;
    AT* dst = (AT*)p.q + ((size_t)row * p.H + hd) * p.D;
    if (hd >= p.H)
      dst = (AT*)(is_v ? p.vc : p.kc) + (((size_t)(slot / p.bs) * p.G + (is_v ? hd - p.H - p.G : hd - p.H)) * p.bs + slot % p.bs) * p.D;
#pragma unroll
    for (int i = 0; i < NP; ++i)
      if (in[i]) ElemIO<AT>::store8(dst + col[i], x[i]);
  };
  auto gains = [&](int hd, float(&g)[NP][8]) {
#pragma unroll
    for (int i = 0; i < NP; ++i) ElemIO<float>::load8(p.gain + min(hd, p.H + p.G - 1) * p.D + col[i], g[i]);
  };

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
    sq = wave_sum(sq);
    sk = wave_sum(sk);
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
    rq = 1.f / sqrtf(sq * p.inv_q + p.eps);
    rk = 1.f / sqrtf(sk * p.inv_k + p.eps);
  }
  // (uniform trip count: the groups of a wave reduce together)
  for (int h0 = blockIdx.z * ng; h0 < heads; h0 += ng * gridDim.z) {
    const int hd = min(h0 + grp, heads - 1);
    const bool on = h0 + grp < heads;
    float gain[NP][8];
    gains(hd, gain);
    if constexpr (K == 4) {
      float b[8], w[4][8], win[4][8];
      bias_of(hd, 0, b);
#pragma unroll
      for (int k = 0; k < 4; ++k) {  // w[k] meets the input 3 - k tokens back
        const int tap = k - (4 - p.taps);
        ElemIO<float>::load8(p.conv + (size_t)max(tap, 0) * C + hd * p.D + col[0], w[k]);
        if (tap < 0) {
#pragma unroll
          for (int j = 0; j < 8; ++j) w[k][j] = 0.f;
        }
      }
#pragma unroll
      for (int k = 1; k < 4; ++k) {  // win[k] = input of token t0 + k - 4
#pragma unroll
        for (int j = 0; j < 8; ++j) win[k][j] = 0.f;
        if (4 - k < p.taps) past(t0, 4 - k, hd, 0, b, win[k]);
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) win[0][j] = 0.f;
      for (int a = 0; a < nt; a += 4) {
        float u[4][8];
#pragma unroll
        for (int i = 0; i < 4; ++i) input(t0 + min(a + i, nt - 1), hd, 0, b, u[i]);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float x[NP][8];
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            win[i][j] = u[i][j];
            x[0][j] = 0.f;
#pragma unroll
            for (int k = 0; k < 4; ++k) x[0][j] = fmaf(w[k][j], win[(i + 1 + k) % 4][j], x[0][j]);
          }
          if (a + i < nt) finish(t0 + a + i, hd, on, x, gain);
        }
      }
    } else {
      for (int t = t0; t < t0 + nt; ++t) {
        float x[NP][8];
#pragma unroll
        for (int i = 0; i < NP; ++i) value(t, hd, i, x[i]);
        finish(t, hd, on, x, gain);
      }
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
  const bool window = p.cu && p.conv && !p.whole && p.taps <= 4 && p.D <= 256;
  const int nt = p.cu && !p.whole ? 8 : 1;
  int bt = 256, slices = 1;
  if (nt == 1) {
    bt = (heads * lph + 63) / 64 * 64;
    const int most = p.cu ? 256 : 1024;
    if (!p.whole && rows < 128 && bt > 256) {  // few decoded tokens: a token's heads over several workgroups
      slices = (bt + 255) / 256;
      bt = 256;
    }
    bt = bt > most ? most : bt;
  }
  const dim3 grid(p.cu ? (max_q + nt - 1) / nt : rows, p.cu ? rows : 1, slices);
#define AI_L(PT, AT, LPH, NP, K, NT, W, CU) \
  hipLaunchKernelGGL((attn_inputs_kernel<PT, AT, LPH, NP, K, NT, W, CU>), grid, dim3(bt), 0, s, p)
#define AI_K(PT, AT, LPH, NP, KW)                                     \
  do {                                                                \
    if (p.cu && p.whole) AI_L(PT, AT, LPH, NP, 0, 1, true, true);     \
    else if (window) AI_L(PT, AT, LPH, NP, KW, 8, false, true);       \
    else if (p.cu) AI_L(PT, AT, LPH, NP, 0, 8, false, true);          \
    else if (p.whole) AI_L(PT, AT, LPH, NP, 0, 1, true, false);       \
    else AI_L(PT, AT, LPH, NP, 0, 1, false, false);                   \
  } while (0)
#define AI_D(PT, AT)                                                                                                \
  do {                                                                                                              \
    if (p.D <= 64) AI_K(PT, AT, 8, 1, 4);                                                                           \
    else if (p.D <= 128) AI_K(PT, AT, 16, 1, 4);                                                                    \
    else if (p.D <= 256) AI_K(PT, AT, 32, 1, 4);                                                                    \
    else AI_K(PT, AT, 64, 2, 0);                                                                                    \
    if (p.cu && p.conv)                                                                                             \
      hipLaunchKernelGGL((attn_ring_kernel<PT, AT>), dim3((C / 8 + 255) / 256, p.taps, rows), dim3(256), 0, s, p);  \
  } while (0)
  DAB_PROJ_DISPATCH(p.y, act_f32, AI_D);
#undef AI_D
#undef AI_K
#undef AI_L
  return hipGetLastError();
}

}  // namespace dab
