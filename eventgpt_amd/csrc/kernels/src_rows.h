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

// RMS norm of `n` columns of a projection row by one wave, stored with zeros up to `ld` columns
template <typename T>
__device__ __forceinline__ void latent_row(const SrcRows& s, long long row, int col, int n, int ld, const float* w, float eps,
                                           T* out, int lane) {
  auto value = [&](int c, float (&v)[8]) {
    if (c + 8 <= n) { src8(s, row, col + c, v); return; }
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = c + i < n ? src1(s, row, col + c + i) : 0.f;
  };
  float v0[8], ss = 0.f;
  for (int c = lane * 8; c < ld; c += 512) {
    float v[8];
    value(c, v);
    ss += sumsq8(v);
    if (c == lane * 8)
#pragma unroll
      for (int i = 0; i < 8; ++i) v0[i] = v[i];
  }
  const float r = rsqrtf(wave_sum(ss) / static_cast<float>(n) + eps);
  for (int c = lane * 8; c < ld; c += 512) {
    float v[8], g[8];
    if (c == lane * 8) {
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = v0[i];
    } else {
      value(c, v);
    }
    load8(w + c, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= r * g[i];
    store8(out + c, v);
  }
}
// Mean (0 for an RMS norm) and reciprocal root of the mean square (of the deviations) of a row of `n` true
// columns, `ld` padded ones, by a block of 256 threads.  keep: the thread's first NC chunks of eight columns, chunk
// (threadIdx.x + k * 256) * 8; far(c, v) gives a chunk past them again.  Padding columns hold zeros.
struct RowStat { float mean, r; };
template <int NC, typename Far>
__device__ __forceinline__ RowStat row_stat(const float (&keep)[NC][8], int n, int ld, float eps, bool layer, float* red,
                                            Far far) {
  const float inv_n = 1.f / static_cast<float>(n);
  float mean = 0.f;
  if (layer) {
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < NC; ++k)
      if (static_cast<int>(threadIdx.x + k * 256) * 8 < ld)
#pragma unroll
        for (int i = 0; i < 8; ++i) s += keep[k][i];
    for (int c = (threadIdx.x + NC * 256) * 8; c < ld; c += 2048) {
      float v[8];
      far(c, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) s += v[i];
    }
    mean = block_sum(s, red) * inv_n;
  }
  float ss = 0.f;
  auto add = [&](int c, const float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float d = layer && c + i >= n ? 0.f : v[i] - mean;
      ss += d * d;
    }
  };
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (threadIdx.x + k * 256) * 8;
    if (c < ld) add(c, keep[k]);
  }
  for (int c = (threadIdx.x + NC * 256) * 8; c < ld; c += 2048) {
    float v[8];
    far(c, v);
    add(c, v);
  }
  return {mean, rsqrtf(block_sum(ss, red) * inv_n + eps)};
}

}  // namespace evgpt
