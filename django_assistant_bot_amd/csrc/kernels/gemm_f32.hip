// 32-bit GEMM  C[b][M,N] = A[b][M,K] . B[b][N,K]^T  on v_mfma_f32_16x16x4_f32 (full fp32 products and
// sums), for the framework's float32 mode.  64 x 64 tiles, 4 waves of 32 x 32, K in steps of 16
// through LDS; batch strides cover the per-head products of latent attention.
#include "common.h"
#include "launchers.h"

namespace dab {

struct GemmF32 {
  const float* A;
  const float* B;
  float* C;
  long lda, ldb, ldc, sa, sb, sc;
  int M, N, K;
  // GROUP: as in gemm_bt_kernel
  const int4* tiles;
  const int* perm;
  int a_div, scatter;
};

template <bool GROUP>
__global__ __launch_bounds__(256) void gemm_f32_kernel(GemmF32 p) {
  constexpr int BK = 16, LD = 20;  // LDS row stride in floats (16-B aligned, rows spread over the banks)
  __shared__ __attribute__((aligned(16))) float as[64 * LD];
  __shared__ __attribute__((aligned(16))) float bs[64 * LD];
  const float* A = p.A + (size_t)blockIdx.z * p.sa;
  const float* B = p.B + (size_t)blockIdx.z * p.sb;
  float* C = p.C + (size_t)blockIdx.z * p.sc;
  int m0 = blockIdx.y * 64;
  const int n0 = blockIdx.x * 64;
  if (GROUP) {
    const int4 t = p.tiles[blockIdx.y];
    if (t.z <= 0) return;  // whole workgroup
    m0 = t.y;
    p.M = t.y + t.z;
    B += (size_t)t.x * p.N * p.K;
  }
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, g = lane >> 4, li = lane & 15;
  const int wm = (w >> 1) * 32, wn = (w & 1) * 32;
  const int row = tid >> 2, kq = (tid & 3) * 4;
  int ar = min(m0 + row, p.M - 1);
  if (GROUP && p.a_div > 0) ar = p.perm[ar] / p.a_div;
  const float* ga = A + (size_t)ar * p.lda + kq;
  const float* gb = B + (size_t)min(n0 + row, p.N - 1) * p.ldb + kq;
  f32x4 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 ra = *reinterpret_cast<const f32x4*>(ga), rb = *reinterpret_cast<const f32x4*>(gb);
  for (int k0 = 0; k0 < p.K; k0 += BK) {
    *reinterpret_cast<f32x4*>(as + row * LD + kq) = ra;
    *reinterpret_cast<f32x4*>(bs + row * LD + kq) = rb;
    __syncthreads();
    if (k0 + BK < p.K) {
      ra = *reinterpret_cast<const f32x4*>(ga + k0 + BK);
      rb = *reinterpret_cast<const f32x4*>(gb + k0 + BK);
    }
#pragma unroll
    for (int s = 0; s < BK / 4; ++s) {
      float a[2], b[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        a[i] = as[(wm + 16 * i + li) * LD + 4 * s + g];
        b[i] = bs[(wn + 16 * i + li) * LD + 4 * s + g];
      }
      // weight rows in the A slot: a lane ends with 4 consecutive columns of one output row
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(b[j], a[i], acc[i][j], 0, 0, 0);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int m = m0 + wm + 16 * i + li;
    if (m >= p.M) continue;
    const size_t mc = GROUP && p.scatter ? p.perm[m] : m;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int n = n0 + wn + 16 * j + 4 * g;
      if (n < p.N) *reinterpret_cast<f32x4*>(C + mc * p.ldc + n) = acc[i][j];  // N % 4 == 0
    }
  }
}

int gemm_f32(const float* A, long lda, long sa, const float* B, long ldb, long sb, float* C, long ldc, long sc, int M,
             int N, int K, int batch, hipStream_t s) {
  if (M <= 0 || N <= 0 || batch <= 0) return 0;
  if (K <= 0 || K % 16 || N % 4 || lda % 4 || ldb % 4 || ldc % 4 || sa % 4 || sb % 4 || sc % 4 || batch > 65535 ||
      (M + 63) / 64 > 65535)
    return hipErrorInvalidValue;
  GemmF32 p{A, B, C, lda, ldb, ldc, sa, sb, sc, M, N, K, nullptr, nullptr, 0, 0};
  hipLaunchKernelGGL(gemm_f32_kernel<false>, dim3((N + 63) / 64, (M + 63) / 64, batch), dim3(256), 0, s, p);
  return hipGetLastError();
}

int gemm_f32_grouped(const float* A, long lda, const float* B, float* C, long ldc, int N, int K, const int* perm, int a_div,
                     int scatter, const void* tiles, int n_tiles, hipStream_t s) {
  if (n_tiles <= 0 || N <= 0) return 0;
  if (K <= 0 || K % 16 || N % 4 || lda % 4 || ldc % 4 || n_tiles > 65535 || !tiles || !perm) return hipErrorInvalidValue;
  GemmF32 p{A, B, C, lda, K, ldc, 0, 0, 0, 0, N, K, (const int4*)tiles, perm, a_div, scatter};
  hipLaunchKernelGGL(gemm_f32_kernel<true>, dim3((N + 63) / 64, n_tiles, 1), dim3(256), 0, s, p);
  return hipGetLastError();
}

}  // namespace dab
