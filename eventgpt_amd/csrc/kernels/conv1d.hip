// Causal per-channel convolution with bias and silu over the rows of a pack of sequences.
//
// The state of a sequence is its last inputs, in a ring of `taps` slots indexed by position % taps: a
// decode step (decode_step.hip) writes the current token's slot, which none of its taps reads, so any
// number of blocks may read a channel while one of them updates it.  A prefill reads the ring for the
// tokens before its first row and writes it afterwards, in a launch of its own.
#include "src_rows.h"

namespace evgpt {

// row_first[row]: first row of the row's sequence in this pack
template <typename T>
__global__ __launch_bounds__(256) void conv_rows_kernel(SrcRows src, int col0, const float* __restrict__ w,
                                                        const float* __restrict__ bias, T* __restrict__ ring,
                                                        T* __restrict__ out, const int* __restrict__ row_slot,
                                                        const int* __restrict__ row_pos,
                                                        const int* __restrict__ row_first, int C, int taps) {
  const long long row = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const long long slot = row_slot[row];
  const int p = row_pos[row];
  const int back = static_cast<int>(row) - row_first[row];   // rows of the sequence before this one
  float acc = bias[c];
  // an input is what a T projection stores, also when it is still in fp32 slabs
  const T cur = from_f32<T>(src1(src, row, col0 + c));
  for (int j = 0; j < taps; ++j) {
    const int d = taps - 1 - j;               // tokens back
    if (p - d < 0) continue;
    float x;
    if (d == 0) x = to_f32(cur);
    else if (d <= back) x = to_f32(from_f32<T>(src1(src, row - d, col0 + c)));
    else x = to_f32(ring[(slot * taps + (p - d) % taps) * C + c]);
    acc += w[static_cast<long long>(c) * taps + j] * x;
  }
  out[row * C + c] = from_f32<T>(acc * sigmoid_f(acc));
}
// The same over the rows of a pack whose projection is stored in T: a thread walks CR rows of eight channels with
// the last inputs in registers; only a sequence's first taps - 1 rows of a pass look into the ring.
constexpr int CR = 16;
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_pack_kernel(const T* __restrict__ src, long long ld, const float* __restrict__ w,
                                                        const float* __restrict__ bias, const T* __restrict__ ring,
                                                        T* __restrict__ out, const int* __restrict__ row_slot,
                                                        const int* __restrict__ row_pos,
                                                        const int* __restrict__ row_first, int rows, int C) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c >= C) return;
  const int r0 = blockIdx.y * CR, r1 = min(r0 + CR, rows);
  float wv[TAPS][8], b[8], win[TAPS][8];            // win[d]: input d rows back
#pragma unroll
  for (int i = 0; i < 8; ++i)
#pragma unroll
    for (int j = 0; j < TAPS; ++j) wv[j][i] = w[static_cast<long long>(c + i) * TAPS + j];
  load8(bias + c, b);
#pragma unroll
  for (int d = 1; d < TAPS; ++d) load8(src + static_cast<long long>(max(r0 - d, 0)) * ld + c, win[d - 1]);
  for (int row = r0; row < r1; ++row) {
#pragma unroll
    for (int d = TAPS - 1; d > 0; --d)
#pragma unroll
      for (int i = 0; i < 8; ++i) win[d][i] = win[d - 1][i];
    load8(src + static_cast<long long>(row) * ld + c, win[0]);
    const int back = row - row_first[row];
    float acc[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] = b[i];
    if (back >= TAPS - 1) {
#pragma unroll
      for (int d = TAPS - 1; d >= 0; --d)
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[i] += wv[TAPS - 1 - d][i] * win[d][i];
    } else {
      const int p = row_pos[row];
      const long long slot = row_slot[row];
#pragma unroll
      for (int d = TAPS - 1; d >= 0; --d) {
        if (p - d < 0) continue;
        float x[8];
        if (d <= back) {
#pragma unroll
          for (int i = 0; i < 8; ++i) x[i] = win[d][i];
        } else {
          load8(ring + (slot * TAPS + (p - d) % TAPS) * C + c, x);
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[i] += wv[TAPS - 1 - d][i] * x[i];
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] *= sigmoid_f(acc[i]);
    store8(out + static_cast<long long>(row) * C + c, acc);
  }
}
template <typename T>
static bool launch_pack(const SrcRows& src, int col0, const float* w, const float* bias, const void* ring, void* out,
                        const int* row_slot, const int* row_pos, const int* row_first, int rows, int C, int taps, hipStream_t st) {
  const dim3 grid((C / 8 + 255) / 256, (rows + CR - 1) / CR);
  if (C % 8 || col0 % 8 || src.nslab != 1 || grid.y > 65535 || taps < 2 || taps > 4) return false;
  const T* p = static_cast<const T*>(src.p) + col0;
#define EVGPT_CONV(TAPS) hipLaunchKernelGGL((conv_pack_kernel<T, TAPS>), grid, dim3(256), 0, st, p, src.ld, w, bias, \
                                            static_cast<const T*>(ring), static_cast<T*>(out), row_slot, row_pos, row_first, rows, C)
  if (taps == 2) EVGPT_CONV(2);
  else if (taps == 3) EVGPT_CONV(3);
  else EVGPT_CONV(4);
#undef EVGPT_CONV
  return true;
}

void launch_conv_rows(const SrcRows& src, int col0, const float* w, const float* bias, void* ring, void* out, bool f32,
                      const int* row_slot, const int* row_pos, const int* row_first, int rows, int C, int taps,
                      hipStream_t st) {
  if ((src.f32 != 0) == f32) {
    if (f32 ? launch_pack<float>(src, col0, w, bias, ring, out, row_slot, row_pos, row_first, rows, C, taps, st)
            : launch_pack<bf16_t>(src, col0, w, bias, ring, out, row_slot, row_pos, row_first, rows, C, taps, st)) return;
  }
  const dim3 grid(rows, (C + 255) / 256);
  if (f32)
    hipLaunchKernelGGL(conv_rows_kernel<float>, grid, dim3(256), 0, st, src, col0, w, bias, static_cast<float*>(ring),
                       static_cast<float*>(out), row_slot, row_pos, row_first, C, taps);
  else
    hipLaunchKernelGGL(conv_rows_kernel<bf16_t>, grid, dim3(256), 0, st, src, col0, w, bias, static_cast<bf16_t*>(ring),
                       static_cast<bf16_t*>(out), row_slot, row_pos, row_first, C, taps);
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
    ring[(slot * taps + (start + i) % taps) * C + c] = from_f32<T>(src1(src, first + i, col0 + c));
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
