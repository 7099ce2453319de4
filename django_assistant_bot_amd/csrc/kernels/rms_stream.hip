// RMS norms around an fp32 residual stream, and the step between a layer's input projection and its attention.
//
//   embed_rms       x = table[id]; h = x / rms(x) * gain
//   rms_residual    x += sublayer output (GEMM rows or split-K slabs) + bias + the token's expert rows
//                   [+ table[id]];  h = x / rms(x) * gain: everything between two layers in one pass.  With ``post``,
//                   output + bias + expert rows pass an RMS norm of their own before they are added; without ``gain``
//                   h is x as it is
//   sigmoid_gate    x *= sigmoid(columns of a projection), a column for every one or (per > 1) for ``per`` of x
//   softcap         cap tanh(y / cap) of the logits
//   qk_rope_write   [q | k | v] columns of a projection -> interleaved rotary positions on q and k, weightless
//                   RMS norm per head, q rows out, k / v into the paged cache
//
// Gains are fp32 and already hold 1 + w where a model stores them around zero.  The mean is over the true
// width; padded columns are zeros.
#include "launchers.h"
#include "proj.h"

namespace dab {

__device__ __forceinline__ float block_total(float v, float* red) {
  v = wave_sum(v);
  const int nw = blockDim.x >> 6;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += red[i];
  return t;
}

struct RmsParams {
  float* x;
  void* h;
  Proj y;                // sublayer output (p null: none)
  const float* bias;     // [cols] or null
  const void* pairs;     // [rows * top, cols] activation type, or null
  int top;
  const int* ids;        // with table: x += table[ids[row]]
  const void* table;     // activation type, or fp32 (table_f32)
  int table_f32;
  const float* post;     // [cols] gain of the norm of what is added, or null
  const float* gain;     // null: h = x
  float inv_n, eps;
  int rows, cols, fresh; // fresh: x starts at zero (embedding)
};

// one workgroup per row; a thread owns 8 columns at (tid + i blockDim) * 8, i < NV
template <typename PT, typename AT, int NV, bool POST>
__global__ __launch_bounds__(256) void rms_residual_kernel(RmsParams p) {
  __shared__ float red[4], red_post[4];
  const int row = blockIdx.x;
  float x[NV][8];
  float ss = 0.f, sp = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] = 0.f;
    if (c >= p.cols) continue;
    if (!POST && !p.fresh) ElemIO<float>::load8(p.x + (size_t)row * p.cols + c, x[i]);
    if (p.y.p) {
      float v[8];
      proj8<PT>(p.y, row, c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += v[j];
    }
    if (p.bias) {
      float v[8];
      ElemIO<float>::load8(p.bias + c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += v[j];
    }
    if (p.pairs) {
      const AT* q = (const AT*)p.pairs + (size_t)row * p.top * p.cols + c;
      for (int k = 0; k < p.top; ++k) {
        float v[8];
        ElemIO<AT>::load8(q + (size_t)k * p.cols, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] += v[j];
      }
    }
    if (POST) {
#pragma unroll
      for (int j = 0; j < 8; ++j) sp = fmaf(x[i][j], x[i][j], sp);
    }
  }
  const float rp = POST ? 1.f / sqrtf(block_total(sp, red_post) * p.inv_n + p.eps) : 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
    if (c >= p.cols) continue;
    float* xr = p.x + (size_t)row * p.cols + c;
    if (POST) {
      float v[8], g[8];
      ElemIO<float>::load8(xr, v);
      ElemIO<float>::load8(p.post + c, g);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] = (p.fresh ? 0.f : v[j]) + x[i][j] * rp * g[j];
    }
    if (p.table) {
      float v[8];
      if (p.table_f32) ElemIO<float>::load8((const float*)p.table + (size_t)p.ids[row] * p.cols + c, v);
      else ElemIO<AT>::load8((const AT*)p.table + (size_t)p.ids[row] * p.cols + c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += v[j];
    }
    ElemIO<float>::store8(xr, x[i]);
    if (!p.gain) {
      if (p.h) ElemIO<AT>::store8((AT*)p.h + (size_t)row * p.cols + c, x[i]);
      continue;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(x[i][j], x[i][j], ss);
  }
  if (!p.gain) return;
  const float r = 1.f / sqrtf(block_total(ss, red) * p.inv_n + p.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
    if (c >= p.cols) continue;
    float g[8];
    ElemIO<float>::load8(p.gain + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) g[j] *= x[i][j] * r;
    ElemIO<AT>::store8((AT*)p.h + (size_t)row * p.cols + c, g);
  }
}

int rms_residual(float* x, void* h, int act_f32, Proj y, const float* bias, const void* pairs, int top, const int* ids,
                 const void* table, int table_f32, const float* post, const float* gain, int n_true, float eps, int rows,
                 int cols, int fresh, hipStream_t s) {
  if (rows <= 0) return 0;
  if (cols <= 0 || cols % 8 || cols > 16384 || !x || (gain && !h) || n_true < 1 || (pairs && top < 1) ||
      (table && !ids) || (post && !y.p && !pairs) || (y.p && (y.S < 1 || y.ld % 8)))
    return hipErrorInvalidValue;
  const int nv8 = cols / 8;
  const int bt = nv8 >= 256 ? 256 : (nv8 + 63) / 64 * 64;
  const int nv = (nv8 + bt - 1) / bt;
  RmsParams p{x, h, y, bias, pairs, top, ids, table, table_f32, post, gain, 1.f / n_true, eps, rows, cols, fresh};
  if (!y.p) p.y.f32 = act_f32;
#define RMS_L(PT, AT, NV)                                                                                      \
  do {                                                                                                         \
    if (post) hipLaunchKernelGGL((rms_residual_kernel<PT, AT, NV, true>), dim3(rows), dim3(bt), 0, s, p);      \
    else hipLaunchKernelGGL((rms_residual_kernel<PT, AT, NV, false>), dim3(rows), dim3(bt), 0, s, p);          \
  } while (0)
#define RMS_NV(PT, AT)                  \
  do {                                  \
    if (nv <= 1) RMS_L(PT, AT, 1);      \
    else if (nv <= 2) RMS_L(PT, AT, 2); \
    else if (nv <= 4) RMS_L(PT, AT, 4); \
    else RMS_L(PT, AT, 8);              \
  } while (0)
  DAB_PROJ_DISPATCH(p.y, act_f32, RMS_NV);
#undef RMS_NV
#undef RMS_L
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------

template <typename PT, typename AT>
__global__ __launch_bounds__(256) void sigmoid_gate_kernel(Proj y, int col0, int per, AT* x, long ldx, int n) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8, t = blockIdx.y;
  if (c >= n) return;
  float g[8], v[8];
  if (per > 1) {
    g[0] = proj_f32<PT>(y, t, col0 + c / per);
#pragma unroll
    for (int j = 1; j < 8; ++j) g[j] = g[0];
  } else {
    proj8<PT>(y, t, col0 + c, g);
  }
  ElemIO<AT>::load8(x + (size_t)t * ldx + c, v);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] /= 1.f + __expf(-g[j]);
  ElemIO<AT>::store8(x + (size_t)t * ldx + c, v);
}

int sigmoid_gate(Proj y, int col0, int per, void* x, long ldx, int act_f32, int n, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (n < 8 || n % 8 || (per > 1 ? per % 8 : per != 1 || col0 % 8) || y.ld % 8 || y.slab % 8 || ldx % 8 || y.S < 1 || T > (1 << 20)) return hipErrorInvalidValue;
  for (int r = 0; r < T; r += 32768) {
    Proj yr = y;
    yr.p = (const char*)y.p + (size_t)r * y.ld * (y.f32 ? 4 : 2);
    const dim3 grid((n / 8 + 255) / 256, T - r < 32768 ? T - r : 32768);
#define SGATE_L(PT, AT) \
  hipLaunchKernelGGL((sigmoid_gate_kernel<PT, AT>), grid, dim3(256), 0, s, yr, col0, per, (AT*)x + (size_t)r * ldx, ldx, n)
    DAB_PROJ_DISPATCH(y, act_f32, SGATE_L);
#undef SGATE_L
  }
  return hipGetLastError();
}

// tanh to fp32 rounding: odd Taylor polynomial near zero, the exp form (no cancellation there) elsewhere
__device__ __forceinline__ float tanh_exact(float x) {
  const float a = fabsf(x), z = x * x;
  if (a < 0.25f) {
    float s = fmaf(z, 8.8632355e-3f, -2.1869489e-2f);
    s = fmaf(z, s, 5.3968254e-2f);
    s = fmaf(z, s, -1.3333333e-1f);
    s = fmaf(z, s, 3.3333333e-1f);
    return x - x * z * s;
  }
  const float t = 1.f - 2.f / (1.f + __expf(2.f * a));
  return x < 0.f ? -t : t;
}

template <typename PT>
__global__ __launch_bounds__(256) void softcap_kernel(Proj y, float cap, float inv, float* __restrict__ out, int n) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8, t = blockIdx.y;
  if (c >= n) return;
  float v[8];
  proj8<PT>(y, t, c, v);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = cap * tanh_exact(v[j] * inv);
  ElemIO<float>::store8(out + (size_t)t * n + c, v);
}

int softcap(Proj y, float cap, float* out, int n, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (n < 8 || n % 8 || y.ld % 8 || y.slab % 8 || y.S < 1 || T > 65535 || !(cap > 0.f)) return hipErrorInvalidValue;
  const dim3 grid((n / 8 + 255) / 256, T);
  if (y.f32) hipLaunchKernelGGL(softcap_kernel<float>, grid, dim3(256), 0, s, y, cap, 1.f / cap, out, n);
  else hipLaunchKernelGGL(softcap_kernel<bf16>, grid, dim3(256), 0, s, y, cap, 1.f / cap, out, n);
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------

struct RopeParams {
  Proj y;
  int col0;              // q heads, then k heads, then v heads from this column, D columns each
  int H, G, D;           // D: padded head width
  int dim;               // true query / key width (RMS statistic)
  int rot;               // rotated dimensions (even)
  const double* freq;    // [rot / 2]
  float inv_dim, eps;
  int norm;              // 1: q and k over their root mean square
  const int* positions;
  const int64_t* slots;
  void* q;               // [T, H, D]
  void* kc;              // [blocks, G, bs, D]
  void* vc;
  int bs, T;
};

// One workgroup per token: the angles once (p * f formed in fp64, so they are exact to fp32 rounding at any position), then
// groups of LPH lanes walk heads, the next head's elements requested under the current one.  A lane owns the elements
// 4 (lane + LPH i) .. + 3, i < NP.
template <typename PT, typename AT, int LPH, int NP>
__global__ __launch_bounds__(512) void qk_rope_kernel(RopeParams p) {
  __shared__ __attribute__((aligned(16))) float2 cs[2 * LPH * NP];
  const int t = blockIdx.x, grp = threadIdx.x / LPH, lane = threadIdx.x % LPH;
  const int ng = blockDim.x / LPH;
  const int heads = p.H + 2 * p.G;
  auto load = [&](int hd, float(&x)[NP][4]) {
    hd = min(hd, heads - 1);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = min(4 * (lane + LPH * i), p.D - 4);
      const PT* s = (const PT*)p.y.p + (size_t)t * p.y.ld + p.col0 + (size_t)hd * p.D + d;
#pragma unroll
      for (int e = 0; e < 4; ++e) x[i][e] = 0.f;
      ElemIO<PT>::add4(s, x[i]);
      int k = 1;
      s += p.y.slab;
      for (; k + 2 <= p.y.S; k += 2, s += 2 * p.y.slab) {
        float a[4] = {0.f, 0.f, 0.f, 0.f};
        ElemIO<PT>::add4(s, x[i]);
        ElemIO<PT>::add4(s + p.y.slab, a);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[i][e] += a[e];
      }
      if (k < p.y.S) ElemIO<PT>::add4(s, x[i]);
    }
  };
  float nx[NP][4];
  load(grp, nx);
  const int64_t slot = p.slots[t];
  const double pos = (double)p.positions[t];
  for (int pr = threadIdx.x; pr < 2 * LPH * NP; pr += blockDim.x) {
    float c = 1.f, s = 0.f;
    if (2 * pr < p.rot) {
      const double turns = pos * p.freq[pr];
      sincos_turn(turns - rint(turns), s, c);
    }
    cs[pr] = make_float2(c, s);
  }
  const size_t blk = slot >= 0 ? (size_t)(slot / p.bs) : 0, off = slot >= 0 ? (size_t)(slot % p.bs) : 0;
  __syncthreads();
  for (int h0 = 0; h0 < heads; h0 += ng) {  // (uniform trip count: the groups of a wave reduce together)
    const int hd = h0 + grp;
    const bool on = hd < heads, is_v = hd >= p.H + p.G;
    float x[NP][4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < NP; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) x[i][e] = ElemIO<AT>::round(nx[i][e]);
    if (h0 + ng < heads) load(hd + ng, nx);
    if (!is_v) {
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(&cs[2 * (lane + LPH * i)]);
        const bool in = 4 * (lane + LPH * i) < p.D;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float u = x[i][2 * e], v = x[i][2 * e + 1];
          x[i][2 * e] = u * w[2 * e] - v * w[2 * e + 1];
          x[i][2 * e + 1] = v * w[2 * e] + u * w[2 * e + 1];
          if (in) ss += x[i][2 * e] * x[i][2 * e] + x[i][2 * e + 1] * x[i][2 * e + 1];
        }
      }
    }
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float r = !is_v && p.norm ? 1.f / sqrtf(ss * p.inv_dim + p.eps) : 1.f;
    if (!on || (hd >= p.H && slot < 0)) continue;
    const int gk = is_v ? hd - p.H - p.G : hd - p.H;
    AT* dst = hd < p.H ? (AT*)p.q + ((size_t)t * p.H + hd) * p.D
                       : (AT*)(is_v ? p.vc : p.kc) + ((blk * p.G + gk) * p.bs + off) * p.D;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = 4 * (lane + LPH * i);
      if (d >= p.D) continue;
#pragma unroll
      for (int e = 0; e < 4; ++e) x[i][e] *= r;
      ElemIO<AT>::store4(dst + d, x[i]);
    }
  }
}

int qk_rope_write(Proj y, int col0, int H, int G, int D, int dim, int rot, const double* freq, float eps, int norm,
                  const int* positions, const int64_t* slots, void* q, void* kc, void* vc, int act_f32, int bs, int T,
                  hipStream_t s) {
  if (T <= 0) return 0;
  if (H < 1 || G < 1 || D < 4 || D % 4 || col0 % 4 || y.ld % 4 || y.slab % 4 || D > 1024 || dim < 1 || dim > D || rot % 2 || rot > dim || rot < 0 || bs < 1 ||
      (rot && !freq) || y.S < 1)
    return hipErrorInvalidValue;
  RopeParams p{y, col0, H, G, D, dim, rot, freq, 1.f / dim, eps, norm, positions, slots, q, kc, vc, bs, T};
  const int bt = T <= 2048 ? 512 : 256;  // decoded tokens: fewer turns of the head loop; prompts: more workgroups a CU
#define ROPE_NP(PT, AT)                                                                                      \
  do {                                                                                                       \
    if (D <= 64) hipLaunchKernelGGL((qk_rope_kernel<PT, AT, 16, 1>), dim3(T), dim3(bt), 0, s, p);            \
    else if (D <= 128) hipLaunchKernelGGL((qk_rope_kernel<PT, AT, 32, 1>), dim3(T), dim3(bt), 0, s, p);      \
    else if (D <= 256) hipLaunchKernelGGL((qk_rope_kernel<PT, AT, 64, 1>), dim3(T), dim3(bt), 0, s, p);      \
    else hipLaunchKernelGGL((qk_rope_kernel<PT, AT, 64, 4>), dim3(T), dim3(bt), 0, s, p);                    \
  } while (0)
  DAB_PROJ_DISPATCH(y, act_f32, ROPE_NP);
#undef ROPE_NP
  return hipGetLastError();
}

}  // namespace dab
