// A projection as its consumers see it: T rows of ``ld`` columns, either the finished output (S == 1) or the
// producing GEMM's split-K slabs (S > 1, ``slab`` elements apart), which the consumer sums in fp32.
#pragma once
#include "common.h"

namespace dab {

template <typename T>
struct ElemIO;
template <>
struct ElemIO<bf16> {
  static __device__ __forceinline__ float load(const bf16* p) { return bf2f(*p); }
  static __device__ __forceinline__ void store(bf16* p, float v) { *p = f2bf(v); }
  static __device__ __forceinline__ float round(float v) { return bf2f(f2bf(v)); }
  static __device__ __forceinline__ float2 load2(const bf16* p) {
    const uint32_t v = *reinterpret_cast<const uint32_t*>(p);
    return make_float2(__uint_as_float(v << 16), __uint_as_float(v & 0xffff0000u));
  }
  static __device__ __forceinline__ void store2(bf16* p, float a, float b) { *reinterpret_cast<uint32_t*>(p) = pack2bf(a, b); }
  static __device__ __forceinline__ void load8(const bf16* p, float (&f)[8]) {
    unpack8(*reinterpret_cast<const u32x4*>(p), f);
  }
  static __device__ __forceinline__ void store8(bf16* p, const float (&f)[8]) { *reinterpret_cast<u32x4*>(p) = pack8(f); }
  static __device__ __forceinline__ void add4(const bf16* p, float (&f)[4]) {
    const u32x2 v = *reinterpret_cast<const u32x2*>(p);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      f[2 * j] += __uint_as_float(v[j] << 16);
      f[2 * j + 1] += __uint_as_float(v[j] & 0xffff0000u);
    }
  }
  static __device__ __forceinline__ void store4(bf16* p, const float (&f)[4]) {
    *reinterpret_cast<u32x2*>(p) = u32x2{pack2bf(f[0], f[1]), pack2bf(f[2], f[3])};
  }
};
template <>
struct ElemIO<float> {
  static __device__ __forceinline__ float load(const float* p) { return *p; }
  static __device__ __forceinline__ void store(float* p, float v) { *p = v; }
  static __device__ __forceinline__ float round(float v) { return v; }
  static __device__ __forceinline__ float2 load2(const float* p) { return *reinterpret_cast<const float2*>(p); }
  static __device__ __forceinline__ void store2(float* p, float a, float b) { *reinterpret_cast<float2*>(p) = make_float2(a, b); }
  static __device__ __forceinline__ void load8(const float* p, float (&f)[8]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = a[j];
      f[4 + j] = b[j];
    }
  }
  static __device__ __forceinline__ void store8(float* p, const float (&f)[8]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{f[4], f[5], f[6], f[7]};
  }
  static __device__ __forceinline__ void add4(const float* p, float (&f)[4]) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] += v[j];
  }
  static __device__ __forceinline__ void store4(float* p, const float (&f)[4]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
  }
};

// element (row, col) in fp32; the slabs' loads are issued four at a time
template <typename PT>
__device__ __forceinline__ float proj_f32(const Proj& p, long row, int col) {
  const PT* q = (const PT*)p.p + row * p.ld + col;
  float v = ElemIO<PT>::load(q);
  int s = 1;
  for (; s + 4 <= p.S; s += 4) {
    float x[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) x[j] = ElemIO<PT>::load(q + (s + j) * p.slab);
#pragma unroll
    for (int j = 0; j < 4; ++j) v += x[j];
  }
  for (; s < p.S; ++s) v += ElemIO<PT>::load(q + s * p.slab);
  return v;
}

// the same rounded to the activation type, like a finished output
template <typename PT, typename AT>
__device__ __forceinline__ float proj_at(const Proj& p, long row, int col) {
  return ElemIO<AT>::round(proj_f32<PT>(p, row, col));
}

// 8 consecutive elements (col % 8 == 0, ld % 8 == 0)
template <typename PT>
__device__ __forceinline__ void proj8(const Proj& p, long row, int col, float (&f)[8]) {
  const PT* q = (const PT*)p.p + row * p.ld + col;
  ElemIO<PT>::load8(q, f);
  int s = 1;
  for (; s + 4 <= p.S; s += 4) {
    SlabVec8<PT> v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j].load(q + (s + j) * p.slab);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j].add_to(f);
  }
  for (; s < p.S; ++s) {
    SlabVec8<PT> v;
    v.load(q + s * p.slab);
    v.add_to(f);
  }
}

// cosine and sine of a whole number of turns' fraction r in [-1/2, 1/2]: the nearest quarter turn is taken off, then the
// Taylor series on [-pi/4, pi/4] to fp32 rounding
__device__ __forceinline__ void sincos_turn(double r, float& sn, float& cs) {
  const double q = rint(4. * r);
  const float a = (float)((r - 0.25 * q) * 6.283185307179586476925), z = a * a;
  float s = fmaf(z, -2.5052108e-8f, 2.7557319e-6f);
  s = fmaf(z, s, -1.9841270e-4f);
  s = fmaf(z, s, 8.3333333e-3f);
  s = fmaf(z, s, -1.6666667e-1f);
  s = fmaf(a * z, s, a);
  float c = fmaf(z, 2.0876757e-9f, -2.7557319e-7f);
  c = fmaf(z, c, 2.4801587e-5f);
  c = fmaf(z, c, -1.3888889e-3f);
  c = fmaf(z, c, 4.1666667e-2f);
  c = fmaf(z, c, -0.5f);
  c = fmaf(z, c, 1.f);
  const int k = (int)q & 3;
  const float s1 = k & 1 ? c : s, c1 = k & 1 ? s : c;
  sn = k & 2 ? -s1 : s1;
  cs = (k == 1 || k == 2) ? -c1 : c1;
}

// log(1 + e^z) = max(z, 0) + log1p(e), e = e^-|z|, with log1p(e) = 2 atanh(s), s = e / (2 + e) <= 1/3, by its power series:
// fp32 rounding for any z, no branch
__device__ __forceinline__ float softplus_f(float z) {
  const float e = __expf(-fabsf(z)), s = e * __builtin_amdgcn_rcpf(2.f + e), q = s * s;
  float p = fmaf(q, 1.f / 13.f, 1.f / 11.f);
  p = fmaf(q, p, 1.f / 9.f);
  p = fmaf(q, p, 1.f / 7.f);
  p = fmaf(q, p, 1.f / 5.f);
  p = fmaf(q, p, 1.f / 3.f);
  return fmaxf(z, 0.f) + 2.f * fmaf(s * q, p, s);
}

// Type dispatch of kernels <projection type, activation type>: bf16 rows, fp32 slabs of a bf16 model, fp32 model.
#define DAB_PROJ_DISPATCH(y, act_f32, CALL)   \
  do {                                        \
    if (act_f32) {                            \
      if (!(y).f32) return hipErrorInvalidValue; \
      CALL(float, float);                     \
    } else if ((y).f32) {                     \
      CALL(float, bf16);                      \
    } else {                                  \
      CALL(bf16, bf16);                       \
    }                                         \
  } while (0)

}  // namespace dab
