// Mixture of experts: routing, the row plan of the grouped GEMMs, and the shared expert's gated activation.
//
//   route        fp32 logits -> softmax over all experts -> the ``top`` largest, weights over their sum (+ 1e-20)
//                times ``scale``; or (sigmoid, raw softmax) the ``top`` largest as they are times ``scale``.  A correction
//                per expert joins the score where the experts are chosen, not in the weight; one wave per token
//   plan         (token, expert) pairs grouped by expert: perm[sorted position] = pair, and the row tiles of
//                the grouped GEMM, each {expert, first sorted position, rows}; one workgroup.  Pairs of identity experts
//                (index >= E) come last and are in no tile
//   shared_glu   silu(gate) up sigmoid(w_sg h) of the expert that every token runs
//
// Which rows an expert gets does not change a row's result, so the order within an expert is left to the
// LDS atomics.
#include "launchers.h"
#include "proj.h"

namespace dab {

template <typename GT, int EI>
__global__ __launch_bounds__(256) void moe_route_kernel(Proj z, int col0, int E, int top, float scale, int scores,
                                                        const float* correction, int* idx, float* wt, int T) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const bool sigmoid = scores == 1;
  float s[EI], w[EI];  // scores as experts are chosen by them, as weights
  float mx = -__builtin_huge_valf();
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    const int e = lane + 64 * i;
    s[i] = e < E ? proj_f32<GT>(z, t, col0 + e) : -__builtin_huge_valf();
    mx = fmaxf(mx, s[i]);
  }
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    s[i] = sigmoid ? 1.f / (1.f + __expf(-s[i])) : __expf(s[i] - mx);
    sum += s[i];
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    const int e = lane + 64 * i;
    w[i] = sigmoid ? s[i] : s[i] / sum;
    s[i] = e < E ? w[i] + (correction ? correction[e] : 0.f) : -__builtin_huge_valf();
  }
  float total = 0.f, mine = 0.f;  // lane k keeps the k-th choice
  int mine_e = 0;
  for (int k = 0; k < top; ++k) {
    float best = -__builtin_huge_valf(), bw = 0.f;
    int be = E;  // (behind every expert: a lane without one left)
#pragma unroll
    for (int i = 0; i < EI; ++i)
      if (s[i] > best) {
        best = s[i];
        bw = w[i];
        be = lane + 64 * i;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oe = __shfl_xor(be, o, 64);
      const float ow = __shfl_xor(bw, o, 64);
      if (ob > best || (ob == best && oe < be)) {
        best = ob;
        be = oe;
        bw = ow;
      }
    }
    total += bw;
    if (lane == k) {
      mine = bw;
      mine_e = be;
    }
#pragma unroll
    for (int i = 0; i < EI; ++i)
      if (be == lane + 64 * i) s[i] = -__builtin_huge_valf();
  }
  if (lane < top) {
    idx[(size_t)t * top + lane] = mine_e;
    wt[(size_t)t * top + lane] = (scores ? mine : mine / (total + 1e-20f)) * scale;
  }
}

int moe_route(Proj z, int col0, int E, int top, float scale, int scores, const float* correction, int* idx, float* wt, int T,
              hipStream_t s) {
  if (T <= 0) return 0;
  if (E < 1 || E > 1024 || top < 1 || top > 64 || top > E || !z.f32 || z.S < 1 || scores < 0 || scores > 2) return hipErrorInvalidValue;
  const dim3 grid((T + 3) / 4);
  if (E <= 64) hipLaunchKernelGGL((moe_route_kernel<float, 1>), grid, dim3(256), 0, s, z, col0, E, top, scale, scores,
                                  correction, idx, wt, T);
  else if (E <= 256) hipLaunchKernelGGL((moe_route_kernel<float, 4>), grid, dim3(256), 0, s, z, col0, E, top, scale, scores,
                                  correction, idx, wt, T);
  else hipLaunchKernelGGL((moe_route_kernel<float, 16>), grid, dim3(256), 0, s, z, col0, E, top, scale, scores,
                                  correction, idx, wt, T);
  return hipGetLastError();
}

// tiles[i] = {expert, first sorted position, rows, 0}; rows 0 past the last tile
__global__ __launch_bounds__(1024) void moe_plan_kernel(const int* __restrict__ idx, int P, int E, int bm, int* perm,
                                                        int4* tiles, int max_tiles) {
  __shared__ int cnt[1025], off[1025], tof[1025];  // entry E: identity experts
  const int tid = threadIdx.x;
  for (int e = tid; e <= E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int i = tid; i < P; i += 1024) atomicAdd(&cnt[min(idx[i], E)], 1);
  __syncthreads();
  if (tid < 64) {  // prefix sums of rows and tiles, 64 experts a step
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + tid;
      const int c = e < E ? cnt[e] : 0, tc = (c + bm - 1) / bm;
      int a = c, b = tc;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int x = __shfl_up(a, o, 64), y = __shfl_up(b, o, 64);
        if (tid >= o) {
          a += x;
          b += y;
        }
      }
      if (e < E) {
        off[e] = base + a - c;
        tof[e] = tbase + b - tc;
      }
      base += __shfl(a, 63, 64);
      tbase += __shfl(b, 63, 64);
    }
    if (tid == 0) {
      off[E] = base;
      tof[E] = tbase;
    }
  }
  __syncthreads();
  for (int e = tid; e < E; e += 1024) {
    const int n = cnt[e];
    for (int k = 0, t = tof[e]; k < n; k += bm, ++t)
      if (t < max_tiles) tiles[t] = make_int4(e, off[e] + k, min(bm, n - k), 0);
  }
  for (int t = tof[E] + tid; t < max_tiles; t += 1024) tiles[t] = make_int4(0, 0, 0, 0);
  __syncthreads();
  for (int i = tid; i < P; i += 1024) perm[atomicAdd(&off[min(idx[i], E)], 1)] = i;
}

int moe_plan(const int* idx, int P, int E, int bm, int* perm, void* tiles, int max_tiles, hipStream_t s) {
  if (P <= 0) return 0;
  if (E < 1 || E > 1024 || bm < 1 || max_tiles < 1) return hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, s, idx, P, E, bm, perm, (int4*)tiles, max_tiles);
  return hipGetLastError();
}

// out[t, 0..F) = silu(gate) up sigmoid(z_sg); gate columns from col0, up columns from col0 + F of a projection
template <typename PT, typename AT>
__global__ __launch_bounds__(256) void shared_glu_kernel(Proj y, int col0, int F, Proj z, int sg_col, AT* out, long ldo) {
  const int t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c >= F) return;
  const float sg = 1.f / (1.f + __expf(-proj_f32<float>(z, t, sg_col)));
  float g[8], u[8];
  proj8<PT>(y, t, col0 + c, g);
  proj8<PT>(y, t, col0 + F + c, u);
#pragma unroll
  for (int j = 0; j < 8; ++j) g[j] = silu_f(ElemIO<AT>::round(g[j])) * ElemIO<AT>::round(u[j]) * sg;
  ElemIO<AT>::store8(out + (size_t)t * ldo + c, g);
}

int shared_glu(Proj y, int col0, int F, Proj z, int sg_col, void* out, long ldo, int act_f32, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (F < 8 || F % 8 || col0 % 8 || y.ld % 8 || ldo % 8 || !z.f32 || y.S < 1 || z.S < 1 || T > (1 << 20)) return hipErrorInvalidValue;
  for (int r = 0; r < T; r += 32768) {
    const int n = T - r < 32768 ? T - r : 32768;
    Proj yr = y, zr = z;
    yr.p = (const char*)y.p + (size_t)r * y.ld * (y.f32 ? 4 : 2);
    zr.p = (const char*)z.p + (size_t)r * z.ld * 4;
    const dim3 grid((F / 8 + 255) / 256, n);
#define SG_L(PT, AT) \
  hipLaunchKernelGGL((shared_glu_kernel<PT, AT>), grid, dim3(256), 0, s, yr, col0, F, zr, sg_col, (AT*)out + (size_t)r * ldo, ldo)
    DAB_PROJ_DISPATCH(y, act_f32, SG_L);
#undef SG_L
  }
  return hipGetLastError();
}

}  // namespace dab
