// Recurrent mixers with a matrix state per head, carried in fp32 from step to step in per-sequence slots.
//
// Two recurrences share every kernel here (S is D x V per head):
//   delta (gated delta rule)    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//                               k, q unit vectors per head (q also times D^-1/2),
//                               g = exp(-A softplus(a + dt_bias)), beta = sigmoid(b)
//   ssd (state-space duality)   S <- exp(-A dt) S + dt B x^T;  o = S^T C + D x,  dt = softplus(dt + dt_bias)
//                               = the delta form with k = B, q = C, v = x, u = dt v
//
// q, k and v first pass a short causal convolution per channel and silu.  Its past inputs live in a ring
// of ``taps`` entries per slot, entry p % taps holding the input of position p: a token writes an entry
// that no token of its own step reads in another workgroup (its own position minus taps), and entries
// before position 0 are never read, so a slot needs no clearing.  A sequence whose step starts at position
// 0 starts from S = 0 without reading the slot.
//
// The state is stored transposed, [slot][head][V][Dp] with Dp = D rounded up to 32 (zeros): a lane holds 4
// consecutive d, 8 lanes a 128-B line of one column.
//
// Step of a prompt portion:  short_conv -> conv_ring_write -> state_scan (or the chunked form) -> gated_norm
// Step of a decoded token:   state_decode (convolution, ring, gates, state, read-out, per-head norm)
#include "launchers.h"
#include "proj.h"

namespace dab {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + __expf(-z)); }

// sum over the 8 lanes that share a column
__device__ __forceinline__ float sum8(float v) {
  v += __shfl_xor(v, 1, 64);
  v += __shfl_xor(v, 2, 64);
  v += __shfl_xor(v, 4, 64);
  return v;
}

// ----------------------------------------------------------------------------------------------
// convolution over a prompt portion

struct ConvParams {
  Proj y;
  int col0, C, taps;
  const float* w;     // [taps, C]
  const float* bias;  // [C] or null
  void* ring;         // [slots, taps, C]
  const int* slot;    // [chunks]
  const int* pos;     // [T]
  const int* cu;      // [chunks + 1]
  void* out;          // [T, C]
  int span;           // tokens a thread walks, whole turns of the window
};

template <typename PT, typename AT, int K>
__global__ __launch_bounds__(256) void short_conv_kernel(ConvParams p) {
  const int b = blockIdx.z, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  const int r0 = p.cu[b], n = p.cu[b + 1] - r0, t0 = blockIdx.y * p.span;
  if (t0 >= n || c >= p.C) return;
  const int pos0 = p.pos[r0];
  const AT* ring = (const AT*)p.ring + (size_t)p.slot[b] * p.taps * p.C;
  float w[K][8], win[K][8], bias[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) bias[j] = 0.f;
  if (p.bias) ElemIO<float>::load8(p.bias + c, bias);
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int tap = k - (K - p.taps);
    ElemIO<float>::load8(p.w + (size_t)max(tap, 0) * p.C + c, w[k]);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      if (tap < 0) w[k][j] = 0.f;
      win[k][j] = 0.f;
    }
  }
  auto token = [&](int t, float(&v)[8]) {  // input of the chunk's token t
    proj8<PT>(p.y, r0 + t, p.col0 + c, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = ElemIO<AT>::round(v[j]);
  };
#pragma unroll
  for (int k = 1; k < K; ++k) {  // the inputs before t0: win[k] = token t0 - (K - k), which may lie before the chunk
    const int t = t0 - (K - k);
    if (K - k > p.taps - 1) continue;
    if (t >= 0) token(t, win[k]);
    else if (pos0 + t >= 0) ElemIO<AT>::load8(ring + (size_t)((pos0 + t) % p.taps) * p.C + c, win[k]);
  }
  // token t0 + i goes to window entry i % K, so nothing is shifted; inputs are requested PF tokens ahead
  constexpr int PF = K < 4 || K > 8 ? 2 : 4;
  static_assert(K % PF == 0, "whole turns of the window");
  const int t1 = min(n, t0 + p.span);
  float nx[PF][8];
#pragma unroll
  for (int i = 0; i < PF; ++i) token(min(t0 + i, t1 - 1), nx[i]);
  for (int t = t0; t < t1; t += K) {
#pragma unroll
    for (int i0 = 0; i0 < K; i0 += PF) {
      if (t + i0 >= t1) break;  // (uniform in the workgroup)
      float in[PF][8];
#pragma unroll
      for (int i = 0; i < PF; ++i)
#pragma unroll
        for (int j = 0; j < 8; ++j) in[i][j] = nx[i][j];
#pragma unroll
      for (int i = 0; i < PF; ++i) token(min(t + i0 + PF + i, t1 - 1), nx[i]);
#pragma unroll
      for (int i = 0; i < PF; ++i) {
        if (t + i0 + i >= t1) break;
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          win[i0 + i][j] = in[i][j];
          o[j] = bias[j];
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) {
#pragma unroll
          for (int k = 0; k < K; ++k) o[j] = fmaf(w[k][j], win[(i0 + i + 1 + k) % K][j], o[j]);
          o[j] = silu_f(o[j]);
        }
        ElemIO<AT>::store8((AT*)p.out + (size_t)(r0 + t + i0 + i) * p.C + c, o);
      }
    }
  }
}

// the last ``taps`` inputs of every chunk into its ring
template <typename PT, typename AT>
__global__ __launch_bounds__(256) void conv_ring_kernel(ConvParams p) {
  const int b = blockIdx.z, c = blockIdx.x * 256 + threadIdx.x;
  const int r0 = p.cu[b], n = p.cu[b + 1] - r0;
  const int t = n - 1 - (int)blockIdx.y;
  if (t < 0 || c >= p.C) return;
  const int at = p.pos[r0] + t;
  AT* ring = (AT*)p.ring + (size_t)p.slot[b] * p.taps * p.C;
  ElemIO<AT>::store(ring + (size_t)(at % p.taps) * p.C + c, proj_at<PT, AT>(p.y, r0 + t, p.col0 + c));
}

int short_conv(Proj y, int col0, int C, int taps, const float* w, const float* bias, void* ring, const int* slot,
               const int* pos, const int* cu, int chunks, int max_q, void* out, int act_f32, hipStream_t s) {
  if (chunks <= 0 || max_q <= 0) return 0;
  if (C < 8 || C % 8 || col0 % 8 || y.ld % 8 || taps < 1 || taps > 16 || y.S < 1 || y.slab % 8 || chunks > 65535 || max_q > (1 << 19))
    return hipErrorInvalidValue;
  // long walks amortise the taps and the inputs before them; short ones keep a single prompt's latency down
  const int wide = (C / 8 + 255) / 256, span = (long)wide * ((max_q + 31) / 32) * chunks >= 1024 ? 32 : taps <= 8 ? 8 : 16;
  ConvParams p{y, col0, C, taps, w, bias, ring, slot, pos, cu, out, span};
  const dim3 grid(wide, (max_q + span - 1) / span, chunks);
#define CONV_K(PT, AT)                                                                                        \
  do {                                                                                                        \
    if (taps <= 2) hipLaunchKernelGGL((short_conv_kernel<PT, AT, 2>), grid, dim3(256), 0, s, p);              \
    else if (taps <= 4) hipLaunchKernelGGL((short_conv_kernel<PT, AT, 4>), grid, dim3(256), 0, s, p);              \
    else if (taps <= 8) hipLaunchKernelGGL((short_conv_kernel<PT, AT, 8>), grid, dim3(256), 0, s, p);         \
    else hipLaunchKernelGGL((short_conv_kernel<PT, AT, 16>), grid, dim3(256), 0, s, p);                       \
    hipLaunchKernelGGL((conv_ring_kernel<PT, AT>), dim3((C + 255) / 256, taps, chunks), dim3(256), 0, s, p);  \
  } while (0)
  DAB_PROJ_DISPATCH(y, act_f32, CONV_K);
#undef CONV_K
  return hipGetLastError();
}

// one decoded token per sequence: 8 channels a thread
template <typename PT, typename AT>
__global__ __launch_bounds__(64) void conv_step_kernel(ConvParams p, int row0, int z_col, AT* z_out) {
  const int b = blockIdx.y, c = (blockIdx.x * 64 + threadIdx.x) * 8, row = row0 + b;
  if (c >= p.C) return;
  const int pos = p.pos[row], now = pos % p.taps;
  AT* ring = (AT*)p.ring + (size_t)p.slot[b] * p.taps * p.C + c;
  float cur[8], o[8], w[8];
  proj8<PT>(p.y, row, p.col0 + c, cur);
  ElemIO<float>::load8(p.w + (size_t)(p.taps - 1) * p.C + c, w);
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = 0.f;
  if (p.bias) ElemIO<float>::load8(p.bias + c, o);
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    cur[j] = ElemIO<AT>::round(cur[j]);
    o[j] = fmaf(w[j], cur[j], o[j]);
  }
  for (int k0 = 1; k0 < p.taps; k0 += 4) {  // four past inputs requested at a time
    float past[4][8], tap[4][8];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int k = k0 + q, e = k < p.taps ? (now >= k ? now - k : now - k + p.taps) : now;
      ElemIO<AT>::load8(ring + (size_t)e * p.C, past[q]);
      ElemIO<float>::load8(p.w + (size_t)(k < p.taps ? p.taps - 1 - k : 0) * p.C + c, tap[q]);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q)
      if (k0 + q < p.taps && k0 + q <= pos) {
#pragma unroll
        for (int j = 0; j < 8; ++j) o[j] = fmaf(tap[q][j], past[q][j], o[j]);
      }
  }
  ElemIO<AT>::store8(ring + (size_t)now * p.C, cur);
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = silu_f(o[j]);
  ElemIO<AT>::store8((AT*)p.out + (size_t)row * p.C + c, o);
  if (z_out) {
    proj8<PT>(p.y, row, z_col + c, o);
    ElemIO<AT>::store8(z_out + (size_t)row * p.C + c, o);
  }
}

int short_conv_step(Proj y, int col0, int C, int taps, const float* w, const float* bias, void* ring, const int* slot,
                    const int* pos, int row0, int B, void* out, int z_col, void* z_out, int act_f32, hipStream_t s) {
  if (B <= 0) return 0;
  if (C < 8 || C % 8 || col0 % 8 || z_col % 8 || y.ld % 8 || taps < 1 || taps > 16 || y.S < 1 || y.slab % 8 || B > 65535) return hipErrorInvalidValue;
  ConvParams p{y, col0, C, taps, w, bias, ring, slot, pos, nullptr, out, 0};
  const dim3 grid((C / 8 + 63) / 64, B);
#define CSTEP_L(PT, AT) hipLaunchKernelGGL((conv_step_kernel<PT, AT>), grid, dim3(64), 0, s, p, row0, z_col, (AT*)z_out)
  DAB_PROJ_DISPATCH(y, act_f32, CSTEP_L);
#undef CSTEP_L
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------
// token-by-token scan of a prompt portion (any sizes, either type)

struct ScanParams {
  const void* conv;   // [T, C] convolved q | k | v (delta) or v | k | q (ssd) columns at q_col / k_col / v_col
  int C, q_col, k_col, v_col;
  int H, G, D, Dp, V;
  Proj gates;         // a (or dt) at a_col, b at b_col
  int a_col, b_col;
  const float* A;     // [H] exp(A_log)
  const float* dt_bias;
  const float* skip;  // ssd: D per head
  float* state;       // [slots, H, V, Dp]
  const int* slot;
  const int* pos;
  const int* cu;
  void* out;          // [T, H * V]
  float qscale;
};

template <typename GT, bool DELTA>
__device__ __forceinline__ void step_gates(const ScanParams& p, long row, int h, float& decay_log, float& beta) {
  const float dt = softplus_f(proj_f32<GT>(p.gates, row, p.a_col + h) + p.dt_bias[h]);
  decay_log = -p.A[h] * dt;
  beta = DELTA ? sigmoid_f(proj_f32<GT>(p.gates, row, p.b_col + h)) : dt;
}

// A wave holds 16 columns: lane = (column c = lane / 8 and c + 8, d quarter lane % 8), DJ float4 each.
template <typename GT, typename AT, int DJ, bool DELTA>
__global__ __launch_bounds__(256) void state_scan_kernel(ScanParams p) {
  constexpr int TB = DJ > 8 ? 8 : 16, Dp = 32 * DJ;
  __shared__ __attribute__((aligned(16))) float ks[TB][Dp];
  __shared__ __attribute__((aligned(16))) float qs[TB][Dp];
  __shared__ float vs[TB][64], gs[TB], bs[TB], rk[TB], rq[TB];
  const int h = blockIdx.y, b = blockIdx.z, hk = h / (p.H / p.G);
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, nw = blockDim.x >> 6, part = lane & 7;
  const int r0 = p.cu[b], n = p.cu[b + 1] - r0;
  if (n <= 0) return;
  const int cols0 = blockIdx.x * 16 * nw;
  float S[2][DJ][4];
  int col[2];
  float* sp[2];
  const bool fresh = p.pos[r0] == 0;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    col[i] = cols0 + w * 16 + (lane >> 3) + 8 * i;
    sp[i] = p.state + (((size_t)p.slot[b] * p.H + h) * p.V + min(col[i], p.V - 1)) * Dp + 4 * part;
#pragma unroll
    for (int j = 0; j < DJ; ++j) {
      const f32x4 v = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(sp[i] + 32 * j);
#pragma unroll
      for (int e = 0; e < 4; ++e) S[i][j][e] = v[e];
    }
  }
  const float skip = p.skip ? p.skip[h] : 0.f;
  for (int t0 = 0; t0 < n; t0 += TB) {
    const int m = min(TB, n - t0);
    __syncthreads();
    for (int i = tid; i < TB * Dp; i += blockDim.x) {
      const int t = i / Dp, d = i % Dp;
      float kv = 0.f, qv = 0.f;
      if (t < m && d < p.D) {
        const AT* src = (const AT*)p.conv + (size_t)(r0 + t0 + t) * p.C + hk * p.D + d;
        kv = ElemIO<AT>::load(src + p.k_col);
        qv = ElemIO<AT>::load(src + p.q_col);
      }
      ks[t][d] = kv;
      qs[t][d] = qv;
    }
    for (int i = tid; i < TB * 16 * nw; i += blockDim.x) {
      const int t = i / (16 * nw), c = i % (16 * nw);
      float v = 0.f;
      if (t < m && cols0 + c < p.V)
        v = ElemIO<AT>::load((const AT*)p.conv + (size_t)(r0 + t0 + t) * p.C + p.v_col + h * p.V + cols0 + c);
      vs[t][c] = v;
    }
    if (tid < m) {
      float dl, be;
      step_gates<GT, DELTA>(p, r0 + t0 + tid, h, dl, be);
      gs[tid] = __expf(dl);
      bs[tid] = be;
    }
    __syncthreads();
    for (int t = w; t < TB; t += nw) {
      float a = 0.f, c = 0.f;
      if (DELTA) {
        for (int d = lane; d < Dp; d += 64) {
          a = fmaf(ks[t][d], ks[t][d], a);
          c = fmaf(qs[t][d], qs[t][d], c);
        }
        a = wave_sum(a);
        c = wave_sum(c);
      }
      if (lane == 0) {
        rk[t] = DELTA ? 1.f / sqrtf(a + 1e-6f) : 1.f;
        rq[t] = DELTA ? p.qscale / sqrtf(c + 1e-6f) : 1.f;
      }
    }
    __syncthreads();
    for (int t = 0; t < m; ++t) {
      const float g = gs[t], beta = bs[t], nk = rk[t], nq = rq[t];
      f32x4 k[DJ];
#pragma unroll
      for (int j = 0; j < DJ; ++j) k[j] = *reinterpret_cast<const f32x4*>(&ks[t][32 * j + 4 * part]);
      float u[2], v[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        v[i] = vs[t][w * 16 + (lane >> 3) + 8 * i];
        float dot = 0.f;
#pragma unroll
        for (int j = 0; j < DJ; ++j)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i][j][e] *= g;
            if (DELTA) dot = fmaf(S[i][j][e], k[j][e], dot);
          }
        u[i] = DELTA ? beta * (v[i] - sum8(dot) * nk) * nk : beta * v[i];
      }
      float o[2] = {0.f, 0.f};
#pragma unroll
      for (int j = 0; j < DJ; ++j) {
        const f32x4 q = *reinterpret_cast<const f32x4*>(&qs[t][32 * j + 4 * part]);
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i][j][e] = fmaf(k[j][e], u[i], S[i][j][e]);
            o[i] = fmaf(S[i][j][e], q[e], o[i]);
          }
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const float r = sum8(o[i]) * nq + skip * v[i];
        if (part == 0 && col[i] < p.V)
          ElemIO<AT>::store((AT*)p.out + (size_t)(r0 + t0 + t) * p.H * p.V + h * p.V + col[i], r);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (col[i] < p.V) {
#pragma unroll
      for (int j = 0; j < DJ; ++j)
        *reinterpret_cast<f32x4*>(sp[i] + 32 * j) = f32x4{S[i][j][0], S[i][j][1], S[i][j][2], S[i][j][3]};
    }
}

#define DAB_DJ_SWITCH(DJV, CALL)   \
  switch (DJV) {                   \
    case 1: CALL(1); break;        \
    case 2: CALL(2); break;        \
    case 3: CALL(3); break;        \
    case 4: CALL(4); break;        \
    case 5: case 6: CALL(6); break; \
    case 7: case 8: CALL(8); break; \
    default: return hipErrorInvalidValue; \
  }

static int check_scan(const RecurrentShape& d, const Proj& gates) {
  if (d.H < 1 || d.G < 1 || d.H % d.G || d.D < 1 || d.V < 1 || d.D > 256 || gates.S < 1 || d.H > 65535) return 1;
  if (d.Dp != recurrent_state_width(d.D)) return 1;
  return 0;
}

int recurrent_state_width(int D) {
  const int j = (D + 31) / 32;
  return 32 * (j <= 4 ? j : j <= 6 ? 6 : 8);
}

static ScanParams scan_params(const void* conv, const RecurrentShape& d, Proj gates, const float* A, const float* dt_bias,
                              const float* skip, float* state, const int* slot, const int* pos, const int* cu, void* out) {
  ScanParams p{};
  p.conv = conv;
  p.C = d.C;
  p.q_col = d.q_col;
  p.k_col = d.k_col;
  p.v_col = d.v_col;
  p.H = d.H;
  p.G = d.G;
  p.D = d.D;
  p.Dp = d.Dp;
  p.V = d.V;
  p.gates = gates;
  p.a_col = d.a_col;
  p.b_col = d.b_col;
  p.A = A;
  p.dt_bias = dt_bias;
  p.skip = skip;
  p.state = state;
  p.slot = slot;
  p.pos = pos;
  p.cu = cu;
  p.out = out;
  p.qscale = 1.f / sqrtf((float)d.D);
  return p;
}

int state_scan(const void* conv, int act_f32, RecurrentShape d, Proj gates, const float* A, const float* dt_bias,
               const float* skip, float* state, const int* slot, const int* pos, const int* cu, int chunks, void* out,
               hipStream_t s) {
  if (chunks <= 0) return 0;
  if (check_scan(d, gates) || chunks > 65535) return hipErrorInvalidValue;
  const ScanParams p = scan_params(conv, d, gates, A, dt_bias, skip, state, slot, pos, cu, out);
  const int nw = d.V >= 64 ? 4 : (d.V + 15) / 16;
  const dim3 grid((d.V + 16 * nw - 1) / (16 * nw), d.H, chunks), block(64 * nw);
#define SCAN_L(DJ)                                                                                              \
  do {                                                                                                          \
    if (act_f32) {                                                                                              \
      if (d.delta) hipLaunchKernelGGL((state_scan_kernel<float, float, DJ, true>), grid, block, 0, s, p);       \
      else hipLaunchKernelGGL((state_scan_kernel<float, float, DJ, false>), grid, block, 0, s, p);              \
    } else {                                                                                                    \
      if (d.delta) hipLaunchKernelGGL((state_scan_kernel<float, bf16, DJ, true>), grid, block, 0, s, p);        \
      else hipLaunchKernelGGL((state_scan_kernel<float, bf16, DJ, false>), grid, block, 0, s, p);               \
    }                                                                                                           \
  } while (0)
  if (!gates.f32) return hipErrorInvalidValue;  // the gates of a recurrence stay in 32 bits
  DAB_DJ_SWITCH(d.Dp / 32, SCAN_L)
#undef SCAN_L
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------
// one decoded token per sequence

struct DecodeStep {
  ScanParams s;
  Proj y;             // input projection: convolution channels at col0, gate (delta) at g_col
  int col0, taps, g_col;
  const float* w;
  const float* bias;
  void* ring;
  const float* norm;  // delta: [V] weight of the per-head output norm
  float eps, out_scale;
  void* out;          // delta: column block of the concatenated activations; ssd: [B, H * V]
  long ldo;
  int pad;            // delta: zero columns after the last head
  int row0;
};

template <typename PT, typename AT, int DJ, bool DELTA>
__global__ __launch_bounds__(256) void state_decode_kernel(DecodeStep a) {
  constexpr int Dp = 32 * DJ;
  const ScanParams& p = a.s;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* ks = sm;
  float* qs = sm + Dp;
  float* vs = sm + 2 * Dp;
  float* os = vs + p.V;
  float* red = os + p.V;  // 8
  const int h = blockIdx.x, b = blockIdx.y, hk = h / (p.H / p.G), row = a.row0 + b;
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, part = lane & 7;
  const int slot = p.slot[b], pos = p.pos[row];
  AT* ring = (AT*)a.ring + (size_t)slot * a.taps * p.C;
  const int now = pos % a.taps;  // ring entry of this token
  for (int i = tid; i < 2 * Dp + p.V; i += 256) {
    int ch = -1;
    if (i < Dp) ch = i < p.D ? p.k_col + hk * p.D + i : -1;
    else if (i < 2 * Dp) ch = i - Dp < p.D ? p.q_col + hk * p.D + i - Dp : -1;
    else ch = p.v_col + h * p.V + i - 2 * Dp;
    float v = 0.f;
    if (ch >= 0) {
      const float cur = proj_at<PT, AT>(a.y, row, a.col0 + ch);
      const float* cw = a.w + ch;
      float acc = fmaf(cw[(size_t)(a.taps - 1) * p.C], cur, a.bias ? a.bias[ch] : 0.f);
      for (int j0 = 1; j0 < a.taps; j0 += 4) {  // four past inputs requested at a time
        float past[4], tap[4];
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int j = j0 + q;
          const bool ok = j < a.taps && j <= pos;
          const int e = ok ? (now >= j ? now - j : now - j + a.taps) : now;
          past[q] = ElemIO<AT>::load(ring + (size_t)e * p.C + ch);
          tap[q] = cw[(size_t)(ok ? a.taps - 1 - j : 0) * p.C];
          if (!ok) past[q] = tap[q] = 0.f;
        }
#pragma unroll
        for (int q = 0; q < 4; ++q) acc = fmaf(tap[q], past[q], acc);
      }
      ElemIO<AT>::store(ring + (size_t)now * p.C + ch, cur);
      v = ElemIO<AT>::round(silu_f(acc));
    }
    sm[i] = v;
  }
  float dl, beta;
  step_gates<float, DELTA>(p, row, h, dl, beta);
  const float g = __expf(dl);
  __syncthreads();
  float nk = 1.f, nq = 1.f;
  if (DELTA) {
    if (w < 2) {
      const float* src = w ? qs : ks;
      float t = 0.f;
      for (int d = lane; d < Dp; d += 64) t = fmaf(src[d], src[d], t);
      t = wave_sum(t);
      if (lane == 0) red[w] = t;
    }
    __syncthreads();
    nk = 1.f / sqrtf(red[0] + 1e-6f);
    nq = p.qscale / sqrtf(red[1] + 1e-6f);
  }
  f32x4 k[DJ], q[DJ];
#pragma unroll
  for (int j = 0; j < DJ; ++j) {
    k[j] = *reinterpret_cast<const f32x4*>(ks + 32 * j + 4 * part);
    q[j] = *reinterpret_cast<const f32x4*>(qs + 32 * j + 4 * part);
  }
  const float skip = p.skip ? p.skip[h] : 0.f;
  float* st = p.state + ((size_t)slot * p.H + h) * p.V * Dp + 4 * part;
  for (int c0 = w * 8 + (lane >> 3); c0 < p.V; c0 += 64) {  // two columns a round: c0, c0 + 32
    f32x4 S[2][DJ];
    const int c1 = c0 + 32;
#pragma unroll
    for (int j = 0; j < DJ; ++j) {
      S[0][j] = S[1][j] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (pos > 0) {
        S[0][j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(st + (size_t)c0 * Dp + 32 * j));
        if (c1 < p.V) S[1][j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(st + (size_t)c1 * Dp + 32 * j));
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int c = i ? c1 : c0;
      const float v = c < p.V ? vs[c] : 0.f;
      float dot = 0.f, o = 0.f;
#pragma unroll
      for (int j = 0; j < DJ; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[i][j][e] *= g;
          if (DELTA) dot = fmaf(S[i][j][e], k[j][e], dot);
        }
      const float u = DELTA ? beta * (v - sum8(dot) * nk) * nk : beta * v;
#pragma unroll
      for (int j = 0; j < DJ; ++j) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[i][j][e] = fmaf(k[j][e], u, S[i][j][e]);
          o = fmaf(S[i][j][e], q[j][e], o);
        }
        if (c < p.V) __builtin_nontemporal_store(S[i][j], reinterpret_cast<f32x4*>(st + (size_t)c * Dp + 32 * j));
      }
      o = sum8(o) * nq + skip * v;
      if (part == 0 && c < p.V) os[c] = o;
    }
  }
  __syncthreads();
  AT* out = (AT*)a.out + (size_t)row * a.ldo + h * p.V;
  if (!DELTA) {
    for (int i = tid; i < p.V; i += 256) ElemIO<AT>::store(out + i, os[i]);
    return;
  }
  float t = 0.f;
  for (int i = tid; i < p.V; i += 256) t = fmaf(os[i], os[i], t);
  t = wave_sum(t);
  if (lane == 0) red[4 + w] = t;
  __syncthreads();
  const float r = a.out_scale / sqrtf((red[4] + red[5] + red[6] + red[7]) / p.V + a.eps);
  for (int i = tid; i < p.V; i += 256)
    ElemIO<AT>::store(out + i, os[i] * r * a.norm[i] * silu_f(proj_f32<PT>(a.y, row, a.g_col + h * p.V + i)));
  if (h == p.H - 1)
    for (int i = tid; i < a.pad; i += 256) ElemIO<AT>::store(out + p.V + i, 0.f);
}

int state_decode(Proj y, int col0, int taps, const float* w, const float* bias, void* ring, int act_f32, RecurrentShape d,
                 Proj gates, const float* A, const float* dt_bias, const float* skip, float* state, const int* slot,
                 const int* pos, int row0, int B, int g_col, const float* norm, float eps, float out_scale, void* out,
                 long ldo, int pad, hipStream_t s) {
  if (B <= 0) return 0;
  if (check_scan(d, gates) || taps < 1 || taps > 16 || B > 65535 || !gates.f32 || y.S < 1 || (d.delta && !norm) || d.V > 8192)
    return hipErrorInvalidValue;
  DecodeStep a{};
  a.s = scan_params(nullptr, d, gates, A, dt_bias, skip, state, slot, pos, nullptr, nullptr);
  a.y = y;
  a.col0 = col0;
  a.taps = taps;
  a.g_col = g_col;
  a.w = w;
  a.bias = bias;
  a.ring = ring;
  a.norm = norm;
  a.eps = eps;
  a.out_scale = out_scale;
  a.out = out;
  a.ldo = ldo;
  a.pad = pad;
  a.row0 = row0;
  const dim3 grid(d.H, B);
  const size_t lds = (2 * d.Dp + 2 * d.V + 16) * sizeof(float);
#define DEC_L2(PT, AT, DJ)                                                                                   \
  do {                                                                                                       \
    if (d.delta) hipLaunchKernelGGL((state_decode_kernel<PT, AT, DJ, true>), grid, dim3(256), lds, s, a);    \
    else hipLaunchKernelGGL((state_decode_kernel<PT, AT, DJ, false>), grid, dim3(256), lds, s, a);           \
  } while (0)
#define DEC_L(DJ)                                 \
  do {                                            \
    if (act_f32) {                                \
      if (!y.f32) return hipErrorInvalidValue;    \
      DEC_L2(float, float, DJ);                   \
    } else if (y.f32) {                           \
      DEC_L2(float, bf16, DJ);                    \
    } else {                                      \
      DEC_L2(bf16, bf16, DJ);                     \
    }                                             \
  } while (0)
  DAB_DJ_SWITCH(d.Dp / 32, DEC_L)
#undef DEC_L
#undef DEC_L2
  return hipGetLastError();
}

// ----------------------------------------------------------------------------------------------
// output gate and norm of a recurrent mixer, over groups of ``part`` channels

struct GatedNorm {
  const void* y;      // [T, n] read-out
  Proj gate;          // gate columns from g_col
  int g_col, n, part;
  int gate_first;     // 1: norm(y silu(gate));  0: norm(y) silu(gate)
  int per_head;       // 1: weight index within the group (shared by the groups)
  const float* w;
  float eps, scale;
  void* out;
  long ldo;
  int pad, row0;      // zero columns after the last channel
  int lanes;          // VEC, part / 8 a power of two below 64: lanes of a group (0: 64)
};

// VEC: part, n and every row and column start are multiples of 8.  One wave per group of up to 512 channels (several
// per workgroup), the whole workgroup on a wider one.
template <typename PT, typename AT, bool VEC>
__global__ __launch_bounds__(256) void gated_norm_kernel(GatedNorm p) {
  constexpr int E = VEC ? 8 : 1;
  __shared__ float red[4];
  const int row = p.row0 + blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  // lanes of one group: a whole workgroup, a wave, or (VEC) the part / 8 lanes a narrow group fills
  const bool wide = p.part > 64 * E;
  const int gl = wide ? 256 : (VEC && p.lanes) ? p.lanes : 64;
  const int per = wide ? 1 : 256 / gl;
  const int grp = blockIdx.x * per + (wide ? 0 : (int)threadIdx.x / gl), i0 = wide ? threadIdx.x : (int)threadIdx.x % gl;
  const int ng = p.n / p.part;
  AT* out = (AT*)p.out + (size_t)row * p.ldo;
  if (blockIdx.x == 0)
    for (int i = threadIdx.x; i < p.pad; i += 256) ElemIO<AT>::store(out + p.n + i, 0.f);
  const bool on = grp < ng;  // (no early exit: the lanes of a wave reduce together)
  const AT* y = (const AT*)p.y + (size_t)row * p.n + (size_t)(on ? grp : 0) * p.part;
  const int c0 = (on ? grp : 0) * p.part;
  auto value = [&](int i, float(&v)[E], float(&g)[E]) {
    if constexpr (VEC) {
      ElemIO<AT>::load8(y + i, v);
      proj8<PT>(p.gate, row, p.g_col + c0 + i, g);
    } else {
      v[0] = ElemIO<AT>::load(y + i);
      g[0] = proj_f32<PT>(p.gate, row, p.g_col + c0 + i);
    }
#pragma unroll
    for (int j = 0; j < E; ++j) g[j] = silu_f(g[j]);
  };
  float ss = 0.f, v[E], g[E];
  for (int i = i0 * E; i < p.part; i += gl * E) {
    value(i, v, g);
#pragma unroll
    for (int j = 0; j < E; ++j) {
      const float x = p.gate_first ? v[j] * g[j] : v[j];
      ss = fmaf(x, x, ss);
    }
  }
  for (int o = (wide ? 64 : gl) / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  if (wide) {
    if (lane == 0) red[w] = ss;
    __syncthreads();
    ss = red[0] + red[1] + red[2] + red[3];
  }
  const float r = p.scale / sqrtf(ss / p.part + p.eps);
  if (!on) return;
  for (int i = i0 * E; i < p.part; i += gl * E) {
    if (wide || gl * E < p.part) value(i, v, g);  // (one step: still in registers)
    float o[E];
#pragma unroll
    for (int j = 0; j < E; ++j) o[j] = v[j] * g[j] * r * p.w[(p.per_head ? 0 : c0) + i + j];
    if constexpr (VEC) ElemIO<AT>::store8(out + c0 + i, o);
    else ElemIO<AT>::store(out + c0 + i, o[0]);
  }
}

int gated_norm(const void* y, int act_f32, Proj gate, int g_col, int n, int part, int gate_first, int per_head,
               const float* w, float eps, float scale, void* out, long ldo, int pad, int row0, int T, hipStream_t s) {
  if (T <= 0) return 0;
  if (n < 1 || part < 1 || n % part || gate.S < 1 || T > (1 << 20)) return hipErrorInvalidValue;
  GatedNorm p{y, gate, g_col, n, part, gate_first, per_head, w, eps, scale, out, ldo, pad, row0, 0};
  const int ng = n / part;
  const bool vec = part % 8 == 0 && g_col % 8 == 0 && gate.ld % 8 == 0 && gate.slab % 8 == 0 && ldo % 8 == 0 &&
                   ((uintptr_t)y | (uintptr_t)out | (uintptr_t)gate.p) % 16 == 0;
  const int pl = part / 8;
  if (vec && pl < 64 && (pl & (pl - 1)) == 0) p.lanes = pl;
  const int e = vec ? 8 : 1, per = part > 64 * e ? 1 : 256 / (p.lanes ? p.lanes : 64);
  // rows in grid.y (65535 limit): walk in slices
  for (int r = 0; r < T; r += 32768) {
    GatedNorm q = p;
    q.row0 = row0 + r;
    const dim3 grid((ng + per - 1) / per, T - r < 32768 ? T - r : 32768);
#define GN_L(PT, AT)                                                                                   \
  do {                                                                                                 \
    if (vec) hipLaunchKernelGGL((gated_norm_kernel<PT, AT, true>), grid, dim3(256), 0, s, q);          \
    else hipLaunchKernelGGL((gated_norm_kernel<PT, AT, false>), grid, dim3(256), 0, s, q);             \
  } while (0)
    DAB_PROJ_DISPATCH(gate, act_f32, GN_L);
#undef GN_L
  }
  return hipGetLastError();
}

}  // namespace dab
