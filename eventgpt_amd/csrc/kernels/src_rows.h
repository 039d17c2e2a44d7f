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

// eight columns of a section of `n` true columns; zeros past them
__device__ __forceinline__ void section8(const SrcRows& s, long long row, int col, int n, int c, float (&v)[8]) {
  if (c + 8 <= n) { src8(s, row, col + c, v); return; }
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = c + i < n ? src1(s, row, col + c + i) : 0.f;
}
// RMS norm of `n` columns of a projection row by one wave, stored with zeros up to `ld` columns
template <typename T>
__device__ __forceinline__ void latent_row(const SrcRows& s, long long row, int col, int n, int ld, const float* w, float eps,
                                           T* out, int lane) {
  float v0[8], ss = 0.f;
  for (int c = lane * 8; c < ld; c += 512) {
    float v[8];
    section8(s, row, col, n, c, v);
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
      section8(s, row, col, n, c, v);
    }
    load8(w + c, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= r * g[i];
    store8(out + c, v);
  }
}
// Mean (0 for an RMS norm) and reciprocal root of the mean square (of the deviations) of a row of `n` true
// columns, `ld` padded ones, by a block of 256 threads.  keep: the thread's first NC chunks of eight columns, chunk
// (threadIdx.x + k * 256) * 8; far(c, v) gives a chunk past them again.  Padding columns hold zeros.  Layer norm: every
// wave takes the squares about its own mean, and the four waves' counts, means and squares are put together.
struct RowStat { float mean, r; };
template <int NC, typename Far>
__device__ __forceinline__ RowStat row_stat(const float (&keep)[NC][8], int n, int ld, float eps, bool layer, float* red,
                                            Far far) {
  auto each = [&](auto f) {
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (threadIdx.x + k * 256) * 8;
      if (c < ld) f(c, keep[k]);
    }
    for (int c = (threadIdx.x + NC * 256) * 8; c < ld; c += 2048) {
      float v[8];
      far(c, v);
      f(c, v);
    }
  };
  if (!layer) {
    float ss = 0.f;
    each([&](int, const float (&v)[8]) { ss += sumsq8(v); });
    return {0.f, rsqrtf(block_sum(ss, red) / static_cast<float>(n) + eps)};
  }
  float s = 0.f, cnt = 0.f;
  each([&](int c, const float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) s += v[i];
    cnt += static_cast<float>(min(max(n - c, 0), 8));
  });
  cnt = wave_sum(cnt);
  const float mw = wave_sum(s) / fmaxf(cnt, 1.f);
  float ss = 0.f;
  each([&](int c, const float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float d = c + i < n ? v[i] - mw : 0.f;
      ss += d * d;
    }
  });
  ss = wave_sum(ss);
  const int wid = threadIdx.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) { red[wid] = cnt; red[4 + wid] = mw; red[8 + wid] = ss; }
  __syncthreads();
  float mean = 0.f, sq = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) mean += red[w] * red[4 + w];
  mean /= static_cast<float>(n);
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    const float d = red[4 + w] - mean;
    sq += red[8 + w] + red[w] * d * d;
  }
  return {mean, rsqrtf(sq / static_cast<float>(n) + eps)};
}

}  // namespace evgpt
