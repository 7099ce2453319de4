// Sublayers whose result passes a gate and a norm before it joins an fp32 residual stream, sums over depth, PolyNorm.
//
//   gated_residual  f = sublayer output (GEMM rows or split-K slabs), or the token's expert rows, of which identity experts
//                   (index >= experts) are weight * stream;  f *= sigmoid(gate columns of a projection + bias);
//                   x = stream + f / rms(f) * post.  At a layer's end also: x is kept as result ``n`` of the depth buffer and
//                   becomes sum_j w[j] * result j (j <= n), of which a part may be there already (``ahead``).  h = x, or x / rms(x) * gain.  Everything between a sublayer's
//                   last projection and the next one's first in one pass
//   depth_ahead     for several layers at once, their sums over the results there are so far: a block of layers reads the
//                   results before it once instead of each layer all of them
//   norm_embed      the same over rows of the embedding table: x = norm(table[id])
//   poly_norm       a N(z) + b N(z^2) + c N(z^3) + e over the first n columns of a projection, N(v) = v / rms(v)
//
// Gains and weights are fp32; means are over the true width, padded columns are zeros.
#include "launchers.h"
#include "proj.h"

namespace dab {

__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int nw = blockDim.x >> 6;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += red[i];
  return t;
}

// one workgroup per row; a thread owns 8 columns at (tid + i blockDim) * 8, i < NV
template <typename PT, typename AT, int NV, bool DEPTH>
__global__ __launch_bounds__(1024) void gated_residual_kernel(GatedResidual p) {
  __shared__ float red[16], red_post[16];
  const int row = blockIdx.x;
  const long yrow = p.ids ? p.ids[row] : row;
  float f[NV][8], s[NV][8], d[NV][8];
  float sp = 0.f, ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) f[i][j] = s[i][j] = d[i][j] = 0.f;
    if (c >= p.cols) continue;
    const size_t at = (size_t)row * p.cols + c;
    if (p.src) ElemIO<float>::load8(p.src + at, s[i]);
    if (p.y.p) proj8<PT>(p.y, yrow, c, f[i]);
    if (p.pairs) {
      const int* idx = p.idx + (size_t)row * p.top;
      const float* wt = p.wt + (size_t)row * p.top;
      const AT* q = (const AT*)p.pairs + (size_t)row * p.top * p.cols + c;
      for (int k0 = 0; k0 < p.top; k0 += 4) {  // four choices requested at a time
        float v[4][8];
#pragma unroll
        for (int u = 0; u < 4; ++u) ElemIO<AT>::load8(q + (size_t)min(k0 + u, p.top - 1) * p.cols, v[u]);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          if (k0 + u >= p.top) break;
          const bool real = idx[k0 + u] < p.experts;  // (an identity expert's row was not written)
          const float w = wt[k0 + u];
#pragma unroll
          for (int j = 0; j < 8; ++j) f[i][j] += real ? v[u][j] : w * s[i][j];
        }
      }
    }
    if (p.g.p) {
      float g[8], b[8];
      proj8<PT>(p.g, row, p.g_col + c, g);
      ElemIO<float>::load8(p.g_bias + c, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[i][j] /= 1.f + __expf(-(g[j] + b[j]));
    }
    if (DEPTH) {
      const float* q = p.depth + at;
      int k = p.from;
      if (p.ahead) ElemIO<float>::load8(p.ahead + at, d[i]);
      for (; k + 4 <= p.n; k += 4) {
        float v[4][8];
#pragma unroll
        for (int u = 0; u < 4; ++u) ElemIO<float>::load8(q + (k + u) * p.depth_stride, v[u]);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int j = 0; j < 8; ++j) d[i][j] = fmaf(p.weights[k + u], v[u][j], d[i][j]);
      }
      for (; k < p.n; ++k) {
        float v[8];
        ElemIO<float>::load8(q + k * p.depth_stride, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) d[i][j] = fmaf(p.weights[k], v[j], d[i][j]);
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) sp = fmaf(f[i][j], f[i][j], sp);
  }
  const float rp = 1.f / sqrtf(block_sum(sp, red_post) * p.inv_n + p.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
    if (c >= p.cols) continue;
    const size_t at = (size_t)row * p.cols + c;
    float g[8];
    ElemIO<float>::load8(p.post + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) s[i][j] += f[i][j] * rp * g[j];
    if (DEPTH) {
      if (p.keep) ElemIO<float>::store8(p.depth + p.n * p.depth_stride + at, s[i]);
      const float w = p.weights[p.n];
#pragma unroll
      for (int j = 0; j < 8; ++j) s[i][j] = fmaf(w, s[i][j], d[i][j]);
    }
    ElemIO<float>::store8(p.x + at, s[i]);
    if (!p.gain) {
      ElemIO<AT>::store8((AT*)p.h + at, s[i]);
      continue;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(s[i][j], s[i][j], ss);
  }
  if (!p.gain) return;
  const float r = 1.f / sqrtf(block_sum(ss, red) * p.inv_n + p.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
    if (c >= p.cols) continue;
    float g[8];
    ElemIO<float>::load8(p.gain + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) g[j] *= s[i][j] * r;
    ElemIO<AT>::store8((AT*)p.h + (size_t)row * p.cols + c, g);
  }
}

int gated_residual(GatedResidual p, int act_f32, int rows, hipStream_t s) {
  if (rows <= 0) return 0;
  if (p.cols <= 0 || p.cols % 8 || p.cols > 16384 || !p.x || !p.h || !p.post || (!p.y.p && !p.pairs) ||
      (p.pairs && (p.top < 1 || !p.idx || !p.wt || !p.src)) || (p.g.p && (!p.g_bias || p.g_col % 8 || p.g.ld % 8 || p.g.S < 1)) ||
      (p.y.p && (p.y.S < 1 || p.y.ld % 8)) || (p.y.p && p.g.p && p.y.f32 != p.g.f32) || p.n < 0 ||
      (p.n && (!p.depth || !p.weights || p.depth_stride % 8 || p.from < 0 || p.from > p.n)))
    return hipErrorInvalidValue;
  const Proj& like = p.y.p ? p.y : p.g;
  if (!like.p) return hipErrorInvalidValue;
  const int nv8 = p.cols / 8;
  // few rows: more threads a row; many: fewer, with two pieces each
  const int bt = nv8 > 512 || (rows < 512 && nv8 > 256) ? (nv8 + 63) / 64 * 64 : nv8 > 256 ? 256 : (nv8 + 63) / 64 * 64;
  const int threads = bt > 1024 ? 1024 : bt, nv = (nv8 + threads - 1) / threads;
#define GR_L(PT, AT, NV)                                                                                        \
  do {                                                                                                          \
    if (p.n) hipLaunchKernelGGL((gated_residual_kernel<PT, AT, NV, true>), dim3(rows), dim3(threads), 0, s, p); \
    else hipLaunchKernelGGL((gated_residual_kernel<PT, AT, NV, false>), dim3(rows), dim3(threads), 0, s, p);    \
  } while (0)
#define GR_NV(PT, AT)              \
  do {                             \
    if (nv <= 1) GR_L(PT, AT, 1);  \
    else GR_L(PT, AT, 2);          \
  } while (0)
  DAB_PROJ_DISPATCH(like, act_f32, GR_NV);
#undef GR_NV
#undef GR_L
  return hipGetLastError();
}

template <int M>
__global__ __launch_bounds__(256) void depth_ahead_kernel(const float* __restrict__ over, long stride, const float* __restrict__ w,
                                                          int n, float* __restrict__ out, long vecs) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= vecs) return;
  f32x4 acc[M];
#pragma unroll
  for (int m = 0; m < M; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float* q = over + i * 4;
  int k = 0;
  for (; k + 4 <= n; k += 4) {
    f32x4 v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) v[u] = *reinterpret_cast<const f32x4*>(q + (k + u) * stride);
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int m = 0; m < M; ++m)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[m][j] = fmaf(w[m * n + k + u], v[u][j], acc[m][j]);
  }
  for (; k < n; ++k) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(q + k * stride);
#pragma unroll
    for (int m = 0; m < M; ++m)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[m][j] = fmaf(w[m * n + k], v[j], acc[m][j]);
  }
#pragma unroll
  for (int m = 0; m < M; ++m) *reinterpret_cast<f32x4*>(out + m * stride + i * 4) = acc[m];
}

int depth_ahead(const float* over, long stride, const float* w, int n, int m, float* out, hipStream_t s) {
  if (stride <= 0) return 0;
  if (stride % 4 || n < 1 || m < 1 || m > 8 || (stride / 4 + 255) / 256 > (1u << 31) - 1) return hipErrorInvalidValue;
  const long vecs = stride / 4;
  const dim3 grid((unsigned)((vecs + 255) / 256));
#define DA_L(M) \
  case M: hipLaunchKernelGGL(depth_ahead_kernel<M>, grid, dim3(256), 0, s, over, stride, w, n, out, vecs); break
  switch (m) {
    DA_L(1);
    DA_L(2);
    DA_L(3);
    DA_L(4);
    DA_L(5);
    DA_L(6);
    DA_L(7);
    DA_L(8);
  }
#undef DA_L
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------

template <typename PT, typename AT, int NV>
__global__ __launch_bounds__(1024) void poly_norm_kernel(Proj y, int n, int cols, float a, float b, float c3, float e, float eps,
                                                         AT* __restrict__ out) {
  __shared__ float red[3][16];
  const int row = blockIdx.x;
  float z[NV][8], m2 = 0.f, m4 = 0.f, m6 = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) z[i][j] = 0.f;
    if (c >= cols) continue;
    proj8<PT>(y, row, c, z[i]);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      z[i][j] = c + j < n ? ElemIO<AT>::round(z[i][j]) : 0.f;
      const float q = z[i][j] * z[i][j], q2 = q * q;
      m2 += q;
      m4 += q2;
      m6 = fmaf(q2, q, m6);
    }
  }
  m2 = wave_sum(m2);
  m4 = wave_sum(m4);
  m6 = wave_sum(m6);
  const int nw = blockDim.x >> 6;
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = m2;
    red[1][threadIdx.x >> 6] = m4;
    red[2][threadIdx.x >> 6] = m6;
  }
  __syncthreads();
  m2 = m4 = m6 = 0.f;
  for (int i = 0; i < nw; ++i) {
    m2 += red[0][i];
    m4 += red[1][i];
    m6 += red[2][i];
  }
  const float inv = 1.f / n;
  a /= sqrtf(fmaf(m2, inv, eps));
  b /= sqrtf(fmaf(m4, inv, eps));
  c3 /= sqrtf(fmaf(m6, inv, eps));
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * 8;
    if (c >= cols) continue;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float v = z[i][j];
      z[i][j] = c + j < n ? fmaf(v, fmaf(v, fmaf(v, c3, b), a), e) : 0.f;
    }
    ElemIO<AT>::store8(out + (size_t)row * cols + c, z[i]);
  }
}

int poly_norm(Proj y, int n, int cols, float a, float b, float c, float e, float eps, void* out, int act_f32, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (n < 1 || cols < n || cols % 8 || cols > 65536 || y.S < 1 || y.ld % 8 || y.slab % 8) return hipErrorInvalidValue;
  const int nv8 = cols / 8;
  // few rows: a thread per 8 columns up to a whole workgroup; many: about four pieces a thread
  const int want = T < 512 ? nv8 : nv8 <= 256 ? nv8 : (nv8 + 3) / 4 < 256 ? 256 : (nv8 + 3) / 4;
  const int bt = want > 1024 ? 1024 : (want + 63) / 64 * 64, nv = (nv8 + bt - 1) / bt;
#define PN_L(PT, AT, NV) \
  hipLaunchKernelGGL((poly_norm_kernel<PT, AT, NV>), dim3(T), dim3(bt), 0, s, y, n, cols, a, b, c, e, eps, (AT*)out)
#define PN_NV(PT, AT)                  \
  do {                                 \
    if (nv <= 1) PN_L(PT, AT, 1);      \
    else if (nv <= 2) PN_L(PT, AT, 2); \
    else if (nv <= 4) PN_L(PT, AT, 4); \
    else PN_L(PT, AT, 8);              \
  } while (0)
  DAB_PROJ_DISPATCH(y, act_f32, PN_NV);
#undef PN_NV
#undef PN_L
  return hipGetLastError();
}

}  // namespace dab
