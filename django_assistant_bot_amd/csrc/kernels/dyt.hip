// Dynamic Tanh (DyT) normalisation around an fp32 residual stream, and the tanh-GELU gate of the 32-bit path.
//
//   DyT(v) = tanh(alpha v) w + b        (one scalar slope, per-channel affine, no reduction over the row)
//
// Because DyT has no row statistic it is purely element-wise, so everything between two projections of
// a sandwich-normed layer is ONE pass over the row:
//     y   = sum of the producing GEMM's split-K slabs (or its single output)
//     x  += DyT_post(y) * ls               (norm after the sublayer, layer scale, residual add; fp32)
//     h   = DyT_next(x)                    (norm before the next sublayer, in the GEMM's input type)
// 2 + 4 + 4 + 2 bytes per element of HBM traffic, where norm / scale / add / norm as separate launches
// would move 26.  A thread owns 8 columns, keeps their parameters in registers and walks rows.
#include "common.h"
#include "launchers.h"

namespace dab {

// tanh to fp32 rounding: odd Taylor polynomial below 1/4, (1 - e^-2|x|) / (1 + e^-2|x|) above
__device__ __forceinline__ float tanh_f(float x) {
  const float a = fabsf(x), s = x * x;
  float q = fmaf(s, 0.021869488536155f, -0.053968253968254f);
  q = fmaf(s, q, 0.133333333333333f);
  q = fmaf(s, q, -0.333333333333333f);
  const float small = fmaf(x * s, q, x);
  const float t = __builtin_amdgcn_exp2f(a * -2.8853900817779268f);
  const float big = copysignf((1.f - t) * __builtin_amdgcn_rcpf(1.f + t), x);
  return a < 0.25f ? small : big;
}

template <typename T>
struct Vec8;
template <>
struct Vec8<bf16> {
  static __device__ __forceinline__ void load(const bf16* p, float (&f)[8]) {
    unpack8(*reinterpret_cast<const u32x4*>(p), f);
  }
  static __device__ __forceinline__ void store(bf16* p, const float (&f)[8]) {
    *reinterpret_cast<u32x4*>(p) = pack8(f);
  }
};
template <>
struct Vec8<float> {
  static __device__ __forceinline__ void load(const float* p, float (&f)[8]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = a[j];
      f[4 + j] = b[j];
    }
  }
  static __device__ __forceinline__ void store(float* p, const float (&f)[8]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{f[4], f[5], f[6], f[7]};
  }
};

// x = table[id] * scale (fp32 residual stream); h = DyT(x)
template <typename T>
__global__ __launch_bounds__(256) void embed_dyt_kernel(float* __restrict__ x, T* __restrict__ h,
                                                        const int* __restrict__ ids, const T* __restrict__ table,
                                                        float scale, float alpha, const float* __restrict__ w,
                                                        const float* __restrict__ b, int rows, int cols, int rpb) {
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
  if (c >= cols) return;
  float wv[8], bv[8];
  Vec8<float>::load(w + c, wv);
  Vec8<float>::load(b + c, bv);
  const int r1 = min(rows, (int)(blockIdx.y + 1) * rpb);
  for (int r = blockIdx.y * rpb; r < r1; ++r) {
    float v[8], o[8];
    Vec8<T>::load(table + (size_t)ids[r] * cols + c, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      v[j] *= scale;
      o[j] = fmaf(tanh_f(alpha * v[j]), wv[j], bv[j]);
    }
    Vec8<float>::store(x + (size_t)r * cols + c, v);
    Vec8<T>::store(h + (size_t)r * cols + c, o);
  }
}

struct DytParams {
  const void* y;     // [S][rows][cols] slabs of the producing projection (YT), summed in fp32
  int S;
  long slab_stride;
  float* x;          // [rows, cols] residual stream, updated in place
  float a_post;      // norm after the sublayer; w_post null: y itself
  const float* w_post;
  const float* b_post;
  const float* ls;   // layer scale, or null
  float a_next;      // norm before the next sublayer; w_next null: no h
  const float* w_next;
  const float* b_next;
  void* h;
  int rows, cols, rpb;
};

template <typename YT, typename HT>
__global__ __launch_bounds__(256) void dyt_residual_kernel(DytParams p) {
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
  if (c >= p.cols) return;
  float wp[8], bp[8], lv[8], wn[8], bn[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) lv[j] = 1.f;
  if (p.w_post) {
    Vec8<float>::load(p.w_post + c, wp);
    Vec8<float>::load(p.b_post + c, bp);
  }
  if (p.ls) Vec8<float>::load(p.ls + c, lv);
  if (p.w_next) {
    Vec8<float>::load(p.w_next + c, wn);
    Vec8<float>::load(p.b_next + c, bn);
  }
  const int r1 = min(p.rows, (int)(blockIdx.y + 1) * p.rpb);
  for (int r = blockIdx.y * p.rpb; r < r1; ++r) {
    const size_t off = (size_t)r * p.cols + c;
    const YT* src = (const YT*)p.y + off;
    float y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, x[8];
    Vec8<float>::load(p.x + off, x);
    int s = 0;
    for (; s + 4 <= p.S; s += 4, src += 4 * p.slab_stride) {
      SlabVec8<YT> v[4];
#pragma unroll
      for (int q = 0; q < 4; ++q) v[q].load(src + q * p.slab_stride);
#pragma unroll
      for (int q = 0; q < 4; ++q) v[q].add_to(y);
    }
    for (; s < p.S; ++s, src += p.slab_stride) {
      SlabVec8<YT> v;
      v.load(src);
      v.add_to(y);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float d = p.w_post ? fmaf(tanh_f(p.a_post * y[j]), wp[j], bp[j]) : y[j];
      x[j] = fmaf(d, lv[j], x[j]);
    }
    Vec8<float>::store(p.x + off, x);
    if (p.w_next) {
      float h[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) h[j] = fmaf(tanh_f(p.a_next * x[j]), wn[j], bn[j]);
      Vec8<HT>::store((HT*)p.h + off, h);
    }
  }
}

// rows per workgroup: enough workgroups to fill the chip, then parameter reuse
static void dyt_grid(int rows, int cols, dim3* grid, dim3* block, int* rpb) {
  const int nv = cols / 8;
  const int bt = nv >= 256 ? 256 : ((nv + 63) / 64) * 64;
  const int gx = (nv + bt - 1) / bt;
  int k = (int)(((long)rows * gx) / 4096);
  *rpb = k < 1 ? 1 : (k > 16 ? 16 : k);
  *grid = dim3(gx, (rows + *rpb - 1) / *rpb);
  *block = dim3(bt);
}

int embed_dyt(float* x, void* h, const int* ids, const void* table, int f32, float scale, float alpha, const float* w,
              const float* b, int rows, int cols, hipStream_t s) {
  if (rows <= 0) return 0;
  if (cols <= 0 || cols % 8) return hipErrorInvalidValue;
  dim3 grid, block;
  int rpb;
  dyt_grid(rows, cols, &grid, &block, &rpb);
  if (f32)
    hipLaunchKernelGGL(embed_dyt_kernel<float>, grid, block, 0, s, x, (float*)h, ids, (const float*)table, scale, alpha,
                       w, b, rows, cols, rpb);
  else
    hipLaunchKernelGGL(embed_dyt_kernel<bf16>, grid, block, 0, s, x, (bf16*)h, ids, (const bf16*)table, scale, alpha, w,
                       b, rows, cols, rpb);
  return hipGetLastError();
}

int dyt_residual(float* x, void* h, int h_f32, const void* y, int y_f32, int S, long slab_stride, float a_post,
                 const float* w_post, const float* b_post, const float* ls, float a_next, const float* w_next,
                 const float* b_next, int rows, int cols, hipStream_t s) {
  if (rows <= 0) return 0;
  if (cols <= 0 || cols % 8 || S < 1 || !x || !y || (w_next && !h)) return hipErrorInvalidValue;
  DytParams p{y, S, slab_stride, x, a_post, w_post, b_post, ls, a_next, w_next, b_next, h, rows, cols, 1};
  dim3 grid, block;
  dyt_grid(rows, cols, &grid, &block, &p.rpb);
  if (y_f32 && h_f32) hipLaunchKernelGGL((dyt_residual_kernel<float, float>), grid, block, 0, s, p);
  else if (y_f32) hipLaunchKernelGGL((dyt_residual_kernel<float, bf16>), grid, block, 0, s, p);
  else if (h_f32) hipLaunchKernelGGL((dyt_residual_kernel<bf16, float>), grid, block, 0, s, p);
  else hipLaunchKernelGGL((dyt_residual_kernel<bf16, bf16>), grid, block, 0, s, p);
  return hipGetLastError();
}

// 32-bit path of the gated MLP: x [rows, 2F] = [gate | up] (+ bias [gate | up]) -> act(gate) up (``act``: GluAct),
// times row_scale[perm[row]] (scale_in: the factor multiplies gate and up instead, before the bias)
__global__ __launch_bounds__(256) void glu_f32_kernel(float* __restrict__ out, long ldo, const float* __restrict__ x,
                                                      long rows, int F, int act, const float* __restrict__ bias,
                                                      const float* __restrict__ row_scale, const int* __restrict__ perm,
                                                      int scale_in) {
  const int fv = F >> 2;
  const long n = rows * fv;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long)gridDim.x * 256) {
    const long r = i / fv;
    const int c = (int)(i - r * fv) * 4;
    f32x4 g = *reinterpret_cast<const f32x4*>(x + r * 2 * F + c);
    f32x4 u = *reinterpret_cast<const f32x4*>(x + r * 2 * F + F + c);
    const float rf = row_scale ? row_scale[perm[r]] : 1.f, rs = scale_in ? 1.f : rf;
    if (scale_in) {
      g *= rf;
      u *= rf;
    }
    if (bias) {
      g += *reinterpret_cast<const f32x4*>(bias + c);
      u += *reinterpret_cast<const f32x4*>(bias + F + c);
    }
    f32x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (act == GLU_RELU ? fmaxf(g[j], 0.f) : act == GLU_GELU ? gelu_tanh_f(g[j]) : silu_f(g[j])) * u[j] * rs;
    *reinterpret_cast<f32x4*>(out + r * ldo + c) = o;
  }
}

int glu_f32(float* out, long ldo, const float* x, long rows, int F, int act, const float* bias, const float* row_scale,
            const int* perm, int scale_in, hipStream_t s) {
  if (rows <= 0) return 0;
  if (F <= 0 || F % 4 || ldo % 4 || (row_scale && !perm)) return hipErrorInvalidValue;
  const long n = rows * (F / 4);
  const unsigned grid = (unsigned)((n + 255) / 256 < 4096 ? (n + 255) / 256 : 4096);
  hipLaunchKernelGGL(glu_f32_kernel, dim3(grid), dim3(256), 0, s, out, ldo, x, rows, F, act, bias, row_scale, perm,
                     scale_in);
  return hipGetLastError();
}

}  // namespace dab
