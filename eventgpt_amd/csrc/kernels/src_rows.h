// Reading rows of a projection (`SrcRows`): one matrix of bf16 or fp32, or fp32 split-K slabs summed on load.
#pragma once
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

// all slabs' loads are issued before the first sum
template <int S> __device__ __forceinline__ void sum_slabs8(const float* p, long long slab, float (&o)[8]) {
  float t[S][8];
#pragma unroll
  for (int k = 0; k < S; ++k) load8(p + k * slab, t[k]);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    o[i] = t[0][i];
#pragma unroll
    for (int k = 1; k < S; ++k) o[i] += t[k][i];
  }
}
// eight consecutive values of a projection row
__device__ __forceinline__ void src8(const SrcRows& s, long long row, int col, float (&o)[8]) {
  if (!s.f32) {
    load8(static_cast<const bf16_t*>(s.p) + row * s.ld + col, o);
    return;
  }
  const float* p = static_cast<const float*>(s.p) + row * s.ld + col;
  if (s.nslab == 1) load8(p, o);
  else if (s.nslab == 2) sum_slabs8<2>(p, s.slab, o);
  else if (s.nslab == 4) sum_slabs8<4>(p, s.slab, o);
  else {
    load8(p, o);
    for (int k = 1; k < s.nslab; ++k) {
      float t[8];
      load8(p + k * s.slab, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] += t[i];
    }
  }
}
__device__ __forceinline__ float src1(const SrcRows& s, long long row, int col) {
  if (!s.f32) return bf16_to_f32(static_cast<const bf16_t*>(s.p)[row * s.ld + col]);
  const float* p = static_cast<const float*>(s.p) + row * s.ld + col;
  if (s.nslab == 4) return p[0] + p[s.slab] + p[2 * s.slab] + p[3 * s.slab];
  float v = p[0];
  for (int k = 1; k < s.nslab; ++k) v += p[k * s.slab];
  return v;
}
// a projected value as a matrix stored in T would hold it
template <typename T> __device__ __forceinline__ float src_t(const SrcRows& s, long long row, int col) {
  return to_f32(from_f32<T>(src1(s, row, col)));
}
__device__ __forceinline__ float sumsq8(const float (&v)[8]) {
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) s += v[i] * v[i];
  return s;
}

}  // namespace evgpt
