// Causal per-channel convolution with bias and silu over the rows of a pack of sequences.
//
// The state of a sequence is its last inputs, in a ring of `taps` slots indexed by position % taps: a
// decode step writes the current token's slot, which none of its taps reads, so any number of blocks
// may read a channel while one of them updates it.  A prefill reads the ring for the tokens before its
// first row and writes it afterwards, in a launch of its own.
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

__device__ __forceinline__ float conv_src(const SrcRows& s, long long row, int col) {
  if (!s.f32) return bf16_to_f32(static_cast<const bf16_t*>(s.p)[row * s.ld + col]);
  const float* p = static_cast<const float*>(s.p) + row * s.ld + col;
  float v = p[0];
  for (int k = 1; k < s.nslab; ++k) v += p[k * s.slab];
  return v;
}

// row_first[row]: first row of the row's sequence in this pack
template <typename T>
__global__ __launch_bounds__(256) void conv_rows_kernel(SrcRows src, int col0, const float* __restrict__ w,
                                                        const float* __restrict__ bias, T* __restrict__ ring,
                                                        T* __restrict__ out, const int* __restrict__ row_slot,
                                                        const int* __restrict__ row_pos,
                                                        const int* __restrict__ row_first, int C, int taps, bool update,
                                                        const int* __restrict__ live) {
  const long long row = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const long long slot = row_slot ? row_slot[row] : row;
  const int p = row_pos[row];
  const int back = row_first ? static_cast<int>(row) - row_first[row] : 0;   // rows of the sequence before this one
  float acc = bias[c];
  // an input is what a T projection stores, also when it is still in fp32 slabs
  const T cur = from_f32<T>(conv_src(src, row, col0 + c));
  for (int j = 0; j < taps; ++j) {
    const int d = taps - 1 - j;               // tokens back
    if (p - d < 0) continue;
    float x;
    if (d == 0) x = to_f32(cur);
    else if (d <= back) x = to_f32(from_f32<T>(conv_src(src, row - d, col0 + c)));
    else x = to_f32(ring[(slot * taps + (p - d) % taps) * C + c]);
    acc += w[static_cast<long long>(c) * taps + j] * x;
  }
  out[row * C + c] = from_f32<T>(acc * sigmoid_f(acc));
  if (update && (live == nullptr || live[row])) ring[(slot * taps + p % taps) * C + c] = cur;
}
void launch_conv_rows(const SrcRows& src, int col0, const float* w, const float* bias, void* ring, void* out, bool f32,
                      const int* row_slot, const int* row_pos, const int* row_first, int rows, int C, int taps,
                      bool update, const int* live, hipStream_t st) {
  const dim3 grid(rows, (C + 255) / 256);
  if (f32)
    hipLaunchKernelGGL(conv_rows_kernel<float>, grid, dim3(256), 0, st, src, col0, w, bias, static_cast<float*>(ring),
                       static_cast<float*>(out), row_slot, row_pos, row_first, C, taps, update, live);
  else
    hipLaunchKernelGGL(conv_rows_kernel<bf16_t>, grid, dim3(256), 0, st, src, col0, w, bias, static_cast<bf16_t*>(ring),
                       static_cast<bf16_t*>(out), row_slot, row_pos, row_first, C, taps, update, live);
}

template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(SrcRows src, int col0, T* __restrict__ ring,
                                                        const int* __restrict__ tails, int C, int taps) {
  const int* t = tails + blockIdx.x * 4;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const long long first = t[0], slot = t[2];
  const int n = t[1], start = t[3];
  for (int i = n > taps ? n - taps : 0; i < n; ++i)
    ring[(slot * taps + (start + i) % taps) * C + c] = from_f32<T>(conv_src(src, first + i, col0 + c));
}
void launch_conv_tail(const SrcRows& src, int col0, void* ring, bool f32, const int* tails, int nseq, int C, int taps,
                      hipStream_t st) {
  const dim3 grid(nseq, (C + 255) / 256);
  if (f32)
    hipLaunchKernelGGL(conv_tail_kernel<float>, grid, dim3(256), 0, st, src, col0, static_cast<float*>(ring), tails, C, taps);
  else
    hipLaunchKernelGGL(conv_tail_kernel<bf16_t>, grid, dim3(256), 0, st, src, col0, static_cast<bf16_t*>(ring), tails, C, taps);
}

}  // namespace evgpt
