// Softmax attention over a paged K / V cache for any head width, either type and any grouping: the form of the
// 32-bit mode and of sizes that the MFMA kernels do not tile.  One wave per (token, query head), 64 keys a
// step with a lane per key for the scores and a lane per value column for the sum; online softmax in fp32.
// ``chunk`` > 0: query i sees keys of its own chunk only, floor(i / chunk) chunk .. i.  ``sink`` (or null)
// joins head h's denominator as one more score.  ``slopes`` (or null): slopes[h] times the distance i - j is taken off the
// score of key j.
#include "launchers.h"
#include "proj.h"

namespace dab {

struct AnyAttn {
  const void* q;        // [T, H, D]
  const void* kc;       // [blocks, G, bs, D]
  const void* vc;
  const int* bt;
  int max_blocks, bs;
  const int* cu;        // [B + 1], or null: token t is sequence t
  const int* ctx;       // [B] cached tokens, the queries included
  int B, H, G, D, chunk;
  float scale, out_scale;
  const float* sink;
  const float* slopes;
  void* out;
  long o_tok;
};

template <typename AT, int NV>
__global__ __launch_bounds__(64) void any_attention_kernel(AnyAttn p) {
  extern __shared__ __attribute__((aligned(16))) float qs[];  // [D], then 64 weights, then 64 row offsets
  float* ps = qs + p.D;
  int* rows = reinterpret_cast<int*>(ps + 64);
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, hk = h / (p.H / p.G);
  int b = t, pos;
  if (p.cu) {
    int lo = 0, hi = p.B - 1;  // the sequence of token t: last b with cu[b] <= t
    while (lo < hi) {
      const int mid = (lo + hi + 1) / 2;
      if (p.cu[mid] <= t) lo = mid;
      else hi = mid - 1;
    }
    b = lo;
    if (t >= p.cu[b + 1]) return;
    pos = p.ctx[b] - (p.cu[b + 1] - t);
  } else {
    pos = p.ctx[b] - 1;
  }
  for (int d = lane; d < p.D; d += 64) qs[d] = ElemIO<AT>::load((const AT*)p.q + ((size_t)t * p.H + h) * p.D + d) * p.scale;
  float acc[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[i] = 0.f;
  float m = -1e30f, l = 0.f;
  if (p.sink) {
    m = p.sink[h];
    l = 1.f;
  }
  const float slope = p.slopes ? p.slopes[h] : 0.f;
  const int first = p.chunk > 0 ? pos / p.chunk * p.chunk : 0;
  for (int k0 = first; k0 <= pos; k0 += 64) {
    const int key = k0 + lane, n = min(64, pos - k0 + 1);
    const int kk = min(key, pos);
    const int row = (p.bt[(size_t)b * p.max_blocks + kk / p.bs] * p.G + hk) * p.bs + kk % p.bs;
    __syncthreads();
    rows[lane] = row;
    float s = 0.f;
    const AT* kr = (const AT*)p.kc + (size_t)row * p.D;
    for (int d = 0; d < p.D; d += 2) {
      const float2 e = ElemIO<AT>::load2(kr + d);
      s = fmaf(qs[d], e.x, s);
      s = fmaf(qs[d + 1], e.y, s);
    }
    s -= slope * (float)(pos - key);
    if (key > pos) s = -__builtin_huge_valf();
    const float mn = fmaxf(m, wave_max(s));
    const float a = __expf(m - mn), w = __expf(s - mn);
    l = l * a + wave_sum(w);
    m = mn;
    ps[lane] = w;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] *= a;
    for (int j = 0; j < n; ++j) {
      const AT* vr = (const AT*)p.vc + (size_t)rows[j] * p.D;
      const float pj = ps[j];
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (lane + 64 * i < p.D) acc[i] = fmaf(pj, ElemIO<AT>::load(vr + lane + 64 * i), acc[i]);
    }
  }
  const float r = p.out_scale / l;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (lane + 64 * i < p.D) ElemIO<AT>::store((AT*)p.out + (size_t)t * p.o_tok + h * p.D + lane + 64 * i, acc[i] * r);
}

int any_attention(const void* q, const void* kc, const void* vc, int f32, const int* bt, int max_blocks, int bs,
                  const int* cu, const int* ctx, int B, int T, int H, int G, int D, int chunk, float scale,
                  const float* sink, const float* slopes, void* out, long o_tok, float out_scale, hipStream_t s) {
  if (T <= 0) return 0;
  if (B < 1 || H < 1 || G < 1 || H % G || D < 2 || D % 2 || D > 1024 || H > 65535 || chunk < 0 || bs < 1) return hipErrorInvalidValue;
  AnyAttn p{q, kc, vc, bt, max_blocks, bs, cu, ctx, B, H, G, D, chunk, scale, out_scale, sink, slopes, out, o_tok};
  const dim3 grid(T, H);
  const size_t lds = (D + 128) * sizeof(float);
#define ANY_NV(AT)                                                                                     \
  do {                                                                                                 \
    if (D <= 128) hipLaunchKernelGGL((any_attention_kernel<AT, 2>), grid, dim3(64), lds, s, p);        \
    else if (D <= 256) hipLaunchKernelGGL((any_attention_kernel<AT, 4>), grid, dim3(64), lds, s, p);   \
    else hipLaunchKernelGGL((any_attention_kernel<AT, 16>), grid, dim3(64), lds, s, p);                \
  } while (0)
  if (f32) ANY_NV(float);
  else ANY_NV(bf16);
#undef ANY_NV
  return hipGetLastError();
}

}  // namespace dab
