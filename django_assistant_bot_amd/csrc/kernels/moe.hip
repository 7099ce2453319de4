// Mixture of experts: routing, the row plan of the grouped GEMMs, and the shared expert's gated activation.
//
//   route        fp32 logits -> softmax over all experts -> the ``top`` largest, weights over their sum (+ 1e-20)
//                times ``scale``; or (sigmoid, raw softmax) the ``top`` largest as they are times ``scale``.  A correction
//                per expert joins the score where the experts are chosen, not in the weight; one wave per token
//   plan         (token, expert) pairs grouped by expert: perm[sorted position] = pair, and the row tiles of
//                the grouped GEMM, each {expert, first sorted position, rows}; one workgroup, or
//                for many pairs three launches.  Pairs of identity experts (index >= E) come last and are in no tile
//   shared_glu   silu(gate) up sigmoid(w_sg h) of the expert that every token runs
//
// Which rows an expert gets does not change a row's result, so the order within an expert is left to the
// LDS atomics.
#include <type_traits>

#include "launchers.h"
#include "proj.h"

namespace dab {

// the largest value of the wave, in every lane (DPP: rows of 16, then the rows)
__device__ __forceinline__ float wave_top(float v) {
  const auto step = [](float x, auto ctrl) {
    const int i = __float_as_int(x);  // (lanes without a source keep their own)
    return fmaxf(x, __int_as_float(__builtin_amdgcn_update_dpp(i, i, decltype(ctrl)::value, 0xf, 0xf, false)));
  };
  v = step(v, std::integral_constant<int, 0xb1>{});   // neighbours
  v = step(v, std::integral_constant<int, 0x4e>{});   // pairs
  v = step(v, std::integral_constant<int, 0x141>{});  // quads, mirrored within 8
  v = step(v, std::integral_constant<int, 0x140>{});  // eights, mirrored within 16
  v = step(v, std::integral_constant<int, 0x142>{});  // a row's last lane to the next row
  v = step(v, std::integral_constant<int, 0x143>{});  // the lower half's last lane to the upper half
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63));
}

template <int EI>
__global__ __launch_bounds__(256) void moe_route_kernel(Proj z, int col0, int E, int top, float scale, int scores,
                                                        const float* correction, int* idx, float* wt, int T) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const bool sigmoid = scores == 1;
  float s[EI], w[EI];  // scores as experts are chosen by them, as weights
  const float* q = (const float*)z.p + (long)t * z.ld + col0;
  int col[EI];
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    col[i] = min(lane + 64 * i, E - 1);
    s[i] = q[col[i]];
    w[i] = correction ? correction[col[i]] : 0.f;
  }
  int k = 1;
  for (; k + 4 <= z.S; k += 4) {  // four slabs requested at a time
    float x[4][EI];
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int i = 0; i < EI; ++i) x[u][i] = q[(k + u) * z.slab + col[i]];
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int i = 0; i < EI; ++i) s[i] += x[u][i];
  }
  for (; k < z.S; ++k)
#pragma unroll
    for (int i = 0; i < EI; ++i) s[i] += q[k * z.slab + col[i]];
  float mx = s[0];
#pragma unroll
  for (int i = 1; i < EI; ++i) mx = fmaxf(mx, s[i]);  // (clamped columns repeat a score)
  mx = wave_top(mx);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    s[i] = sigmoid ? 1.f / (1.f + __expf(-s[i])) : __expf(s[i] - mx);
    sum += lane + 64 * i < E ? s[i] : 0.f;
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < EI; ++i) {
    const float c = w[i];
    w[i] = sigmoid ? s[i] : s[i] / sum;
    s[i] = lane + 64 * i < E ? w[i] + c : -__builtin_huge_valf();
  }
  float total = 0.f, mine = 0.f;  // lane k keeps the k-th choice
  int mine_e = 0;
  for (k = 0; k < top; ++k) {
    float best = s[0];
#pragma unroll
    for (int i = 1; i < EI; ++i) best = fmaxf(best, s[i]);
    best = wave_top(best);
    int be = E, at = 0;  // (E: no score is a number)
    float bw = 0.f;
#pragma unroll
    for (int i = EI - 1; i >= 0; --i) {  // the lowest of equal ones
      const unsigned long long m = __ballot(s[i] == best);
      if (m) {
        at = __ffsll(m) - 1;
        be = at + 64 * i;
        bw = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(w[i]), at));
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
#define ROUTE_L(EI) \
  hipLaunchKernelGGL(moe_route_kernel<EI>, grid, dim3(256), 0, s, z, col0, E, top, scale, scores, correction, idx, wt, T)
  if (E <= 64) ROUTE_L(1);
  else if (E <= 128) ROUTE_L(2);
  else if (E <= 256) ROUTE_L(4);
  else ROUTE_L(16);
#undef ROUTE_L
  return hipGetLastError();
}

// Offsets of the experts' rows and tiles from their counts cnt[0 .. E] (entry E: identity experts), by the first wave
__device__ __forceinline__ void plan_offsets(const int* cnt, int* off, int* tof, int E, int bm) {
  const int lane = threadIdx.x;
  int base = 0, tbase = 0;
  for (int e0 = 0; e0 < E; e0 += 64) {
    const int e = e0 + lane;
    const int c = e < E ? cnt[e] : 0, tc = (c + bm - 1) / bm;
    int a = c, b = tc;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int x = __shfl_up(a, o, 64), y = __shfl_up(b, o, 64);
      if (lane >= o) {
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
  if (lane == 0) {
    off[E] = base;
    tof[E] = tbase;
  }
}

// tiles[i] = {expert, first sorted position, rows, 0}; rows 0 past the last tile
__device__ __forceinline__ void plan_tiles(const int* cnt, const int* off, const int* tof, int E, int bm, int4* tiles, int max_tiles) {
  for (int e = threadIdx.x; e < E; e += 1024) {
    const int n = cnt[e];
    for (int k = 0, t = tof[e]; k < n; k += bm, ++t)
      if (t < max_tiles) tiles[t] = make_int4(e, off[e] + k, min(bm, n - k), 0);
  }
  for (int t = tof[E] + threadIdx.x; t < max_tiles; t += 1024) tiles[t] = make_int4(0, 0, 0, 0);
}

__global__ __launch_bounds__(1024) void moe_plan_kernel(const int* __restrict__ idx, int P, int E, int bm, int* perm,
                                                        int4* tiles, int max_tiles) {
  __shared__ int cnt[1025], off[1025], tof[1025];
  const int tid = threadIdx.x;
  for (int e = tid; e <= E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int i = tid; i < P; i += 1024) atomicAdd(&cnt[min(idx[i], E)], 1);
  __syncthreads();
  if (tid < 64) plan_offsets(cnt, off, tof, E, bm);
  __syncthreads();
  plan_tiles(cnt, off, tof, E, bm, tiles, max_tiles);
  __syncthreads();
  for (int i = tid; i < P; i += 1024) perm[atomicAdd(&off[min(idx[i], E)], 1)] = i;
}

// The same for many pairs in three launches: kPlanParts workgroups count their parts, one turns the counts ws[part][E + 1] into
// each part's first positions and writes the tiles, and the parts place their pairs.
constexpr int kPlanParts = 32;

__global__ __launch_bounds__(1024) void moe_count_kernel(const int* __restrict__ idx, int P, int E, int part, int* __restrict__ ws) {
  __shared__ int cnt[1025];
  for (int e = threadIdx.x; e <= E; e += 1024) cnt[e] = 0;
  __syncthreads();
  const int i1 = min(P, (int)(blockIdx.x + 1) * part);
  for (int i = blockIdx.x * part + threadIdx.x; i < i1; i += 1024) atomicAdd(&cnt[min(idx[i], E)], 1);
  __syncthreads();
  for (int e = threadIdx.x; e <= E; e += 1024) ws[blockIdx.x * (E + 1) + e] = cnt[e];
}

__global__ __launch_bounds__(1024) void moe_offsets_kernel(int* __restrict__ ws, int E, int bm, int4* tiles, int max_tiles) {
  __shared__ int cnt[1025], off[1025], tof[1025];
  const int tid = threadIdx.x;
  for (int e = tid; e <= E; e += 1024) {
    int n = 0;
#pragma unroll
    for (int b = 0; b < kPlanParts; ++b) n += ws[b * (E + 1) + e];
    cnt[e] = n;
  }
  __syncthreads();
  if (tid < 64) plan_offsets(cnt, off, tof, E, bm);
  __syncthreads();
  plan_tiles(cnt, off, tof, E, bm, tiles, max_tiles);
  for (int e = tid; e <= E; e += 1024) {
    int n[kPlanParts], at = off[e];
#pragma unroll
    for (int b = 0; b < kPlanParts; ++b) n[b] = ws[b * (E + 1) + e];
#pragma unroll
    for (int b = 0; b < kPlanParts; ++b) {
      ws[b * (E + 1) + e] = at;
      at += n[b];
    }
  }
}

__global__ __launch_bounds__(1024) void moe_place_kernel(const int* __restrict__ idx, int P, int E, int part, const int* __restrict__ ws,
                                                         int* __restrict__ perm) {
  __shared__ int off[1025];
  for (int e = threadIdx.x; e <= E; e += 1024) off[e] = ws[blockIdx.x * (E + 1) + e];
  __syncthreads();
  const int i1 = min(P, (int)(blockIdx.x + 1) * part);
  for (int i = blockIdx.x * part + threadIdx.x; i < i1; i += 1024) perm[atomicAdd(&off[min(idx[i], E)], 1)] = i;
}

int moe_plan_words(int P, int E) { return P < 16384 ? 0 : kPlanParts * (E + 1); }

int moe_plan(const int* idx, int P, int E, int bm, int* perm, void* tiles, int max_tiles, int* ws, hipStream_t s) {
  if (P <= 0) return 0;
  if (E < 1 || E > 1024 || bm < 1 || max_tiles < 1) return hipErrorInvalidValue;
  if (!moe_plan_words(P, E)) {
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, s, idx, P, E, bm, perm, (int4*)tiles, max_tiles);
    return hipGetLastError();
  }
  if (!ws) return hipErrorInvalidValue;
  const int part = (P + kPlanParts - 1) / kPlanParts;
  hipLaunchKernelGGL(moe_count_kernel, dim3(kPlanParts), dim3(1024), 0, s, idx, P, E, part, ws);
  hipLaunchKernelGGL(moe_offsets_kernel, dim3(1), dim3(1024), 0, s, ws, E, bm, (int4*)tiles, max_tiles);
  hipLaunchKernelGGL(moe_place_kernel, dim3(kPlanParts), dim3(1024), 0, s, idx, P, E, part, ws, perm);
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
