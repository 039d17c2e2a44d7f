// Element-type helpers of the layered decoder kernels: every kernel is a template over the storage
// type T of weights and activations -- bf16_t (serving) or float (true 32-bit) -- and computes in fp32.
#pragma once
#include "common.h"

namespace evgpt {

__device__ __forceinline__ float to_f32(bf16_t v) { return bf16_to_f32(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
template <typename T> __device__ __forceinline__ T from_f32(float v);
template <> __device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) { return f32_to_bf16(v); }
template <> __device__ __forceinline__ float from_f32<float>(float v) { return v; }

__device__ __forceinline__ void load8(const bf16_t* p, float (&o)[8]) {
  const u32x4_t w = load16(p);
#pragma unroll
  for (int i = 0; i < 4; ++i) { o[2 * i] = bf16lo(w[i]); o[2 * i + 1] = bf16hi(w[i]); }
}
__device__ __forceinline__ void load8(const float* p, float (&o)[8]) {
  const f32x4_t a = *reinterpret_cast<const f32x4_t*>(p), b = *reinterpret_cast<const f32x4_t*>(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) { o[i] = a[i]; o[4 + i] = b[i]; }
}
__device__ __forceinline__ void store8(bf16_t* p, const float (&v)[8]) {
  *reinterpret_cast<u32x4_t*>(p) = u32x4_t{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                                           pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7])};
}
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
  *reinterpret_cast<f32x4_t*>(p) = f32x4_t{v[0], v[1], v[2], v[3]};
  *reinterpret_cast<f32x4_t*>(p + 4) = f32x4_t{v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ void store4(bf16_t* p, float a, float b, float c, float d) {
  *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack_bf16x2(a, b), pack_bf16x2(c, d)};
}
__device__ __forceinline__ void store4(float* p, float a, float b, float c, float d) {
  *reinterpret_cast<f32x4_t*>(p) = f32x4_t{a, b, c, d};
}
__device__ __forceinline__ f32x4_t load4(const bf16_t* p) {
  const u32x2_t w = *reinterpret_cast<const u32x2_t*>(p);
  return f32x4_t{bf16lo(w[0]), bf16hi(w[0]), bf16lo(w[1]), bf16hi(w[1])};
}
__device__ __forceinline__ f32x4_t load4(const float* p) { return *reinterpret_cast<const f32x4_t*>(p); }

// A 16-row x 32-deep MFMA operand: lane l holds row l % 16, contraction slots (l / 16) * 8 .. + 7.
// float: the same eight slots go through eight 16x16x4 fp32 MFMAs, one slot of every lane group each,
// so both storage types share one register layout (and the accumulator layout: column l % 16, rows
// (l / 16) * 4 + r).
template <typename T> struct Frag;
template <> struct Frag<bf16_t> { bf16x8_t v; };
template <> struct Frag<float> { float v[8]; };

__device__ __forceinline__ Frag<bf16_t> load_frag(const bf16_t* p) {
  return {__builtin_bit_cast(bf16x8_t, load16(p))};
}
__device__ __forceinline__ Frag<float> load_frag(const float* p) {
  Frag<float> f;
  load8(p, f.v);
  return f;
}
__device__ __forceinline__ Frag<bf16_t> zero_frag(bf16_t) { return {__builtin_bit_cast(bf16x8_t, u32x4_t{0, 0, 0, 0})}; }
__device__ __forceinline__ Frag<float> zero_frag(float) { return {{0, 0, 0, 0, 0, 0, 0, 0}}; }

__device__ __forceinline__ f32x4_t mma(const Frag<bf16_t>& a, const Frag<bf16_t>& b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4_t mma(const Frag<float>& a, const Frag<float>& b, f32x4_t c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[j], b.v[j], c, 0, 0, 0);
  return c;
}

// An fp32 operand next to a T operand.  bf16: the fp32 values go in as the sum of two bf16 numbers
// (16 mantissa bits), two MFMAs per product, so that fp32 quantities -- recurrent states, decay
// weights, gated values -- are not rounded to bf16 on their way into the matrix cores.
template <typename T> struct WideFrag;
template <> struct WideFrag<bf16_t> { bf16x8_t hi, lo; };
template <> struct WideFrag<float> { float v[8]; };

template <typename T> __device__ __forceinline__ WideFrag<T> wide_frag(const float (&x)[8]);
template <> __device__ __forceinline__ WideFrag<bf16_t> wide_frag<bf16_t>(const float (&x)[8]) {
  u32x4_t h, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack_bf16x2(x[2 * i], x[2 * i + 1]);
    l[i] = pack_bf16x2(x[2 * i] - bf16lo(h[i]), x[2 * i + 1] - bf16hi(h[i]));
  }
  return {__builtin_bit_cast(bf16x8_t, h), __builtin_bit_cast(bf16x8_t, l)};
}
template <> __device__ __forceinline__ WideFrag<float> wide_frag<float>(const float (&x)[8]) {
  WideFrag<float> f;
#pragma unroll
  for (int i = 0; i < 8; ++i) f.v[i] = x[i];
  return f;
}
__device__ __forceinline__ f32x4_t mma(const WideFrag<bf16_t>& a, const Frag<bf16_t>& b, f32x4_t c) {
  c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.lo, b.v, c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.hi, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4_t mma(const Frag<bf16_t>& a, const WideFrag<bf16_t>& b, f32x4_t c) {
  c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.lo, c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.hi, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4_t mma(const WideFrag<float>& a, const Frag<float>& b, f32x4_t c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[j], b.v[j], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ f32x4_t mma(const Frag<float>& a, const WideFrag<float>& b, f32x4_t c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[j], b.v[j], c, 0, 0, 0);
  return c;
}

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float gelu_tanh_f(float x) {
  return 0.5f * x * (1.f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
}
__device__ __forceinline__ float soft_cap(float x, float scale, float cap) {
  x *= scale;
  return cap > 0.f ? cap * tanhf(x / cap) : x;
}

}  // namespace evgpt
