// True fp32 matrix product  C[M,N] = A[M,K] · W[N,K]^T  on v_mfma_f32_16x16x4_f32 (CDNA4 has no
// reduced-precision fp32 mode to fall into): the products of the layered decoders' 32-bit mode.
// 64 x 64 tile, four waves of 32 x 32, K staged through LDS 32 at a time.  K % 32 == 0.  GROUPED: the rows are sorted
// into groups, each with a weight matrix of its own (experts), and are read through a permutation.
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

constexpr int GF_LD = 36;   // floats per LDS row (32 + 4: rows land on different banks)

struct GroupArgs { const int* start; const int* perm; int top, groups; };

template <bool GROUPED>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const float* __restrict__ A, const float* __restrict__ W,
                                                       float* __restrict__ C, int M, int N, int K, int lda, int ldw,
                                                       int ldc, GroupArgs grp) {
  __shared__ __attribute__((aligned(16))) float sa[64 * GF_LD], sw[64 * GF_LD];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int fr = lane & 15, g = lane >> 4;
  int n0 = blockIdx.x * 64, m0 = blockIdx.y * 64, first = 0;
  if constexpr (GROUPED) {
    const int tiles_n = (N + 63) / 64;
    int tile = blockIdx.x;
    const int e = group_of_tile(grp.start, grp.groups, 64, tiles_n, tile);
    if (e < 0) return;
    first = grp.start[e];
    M = grp.start[e + 1] - first;
    m0 = tile / tiles_n * 64;
    n0 = tile % tiles_n * 64;
    W += static_cast<long long>(e) * N * ldw;
    C += static_cast<long long>(first) * ldc;
  }
  // source row of tile row m
  auto row_of = [&](int m) {
    m = min(m, M - 1);
    if constexpr (GROUPED) return grp.perm ? grp.perm[first + m] / grp.top : first + m;
    return m;
  };
  int arow[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) arow[i] = row_of(m0 + ((tid + i * 256) >> 3));
  const int wm = (wid >> 1) * 32, wn = (wid & 1) * 32;
  f32x4_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += 32) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i) {      // 64 rows x 8 four-float chunks per operand
      const int idx = tid + i * 256, row = idx >> 3, ch = (idx & 7) * 4;
      const int am = arow[i], wr = min(n0 + row, N - 1);
      *reinterpret_cast<f32x4_t*>(sa + row * GF_LD + ch) = load4(A + static_cast<size_t>(am) * lda + k0 + ch);
      *reinterpret_cast<f32x4_t*>(sw + row * GF_LD + ch) = load4(W + static_cast<size_t>(wr) * ldw + k0 + ch);
    }
    __syncthreads();
    Frag<float> a[2], w[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      a[i] = load_frag(sa + (wm + i * 16 + fr) * GF_LD + g * 8);
      w[i] = load_frag(sw + (wn + i * 16 + fr) * GF_LD + g * 8);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = mma(w[j], a[i], acc[i][j]);   // rows: output columns, lane: token
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int m = m0 + wm + i * 16 + fr;
    if (m >= M) continue;
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = n0 + wn + j * 16 + g * 4 + r;
        if (n < N) C[static_cast<size_t>(m) * ldc + n] = acc[i][j][r];
      }
  }
}

void launch_gemm_f32(const float* A, const float* W, float* C, int M, int N, int K, int lda, int ldw, int ldc,
                     hipStream_t st) {
  hipLaunchKernelGGL(gemm_f32_kernel<false>, dim3((N + 63) / 64, (M + 63) / 64), dim3(256), 0, st, A, W, C, M, N, K, lda, ldw,
                     ldc, GroupArgs{});
}
void launch_gemm_f32_grouped(const float* A, const float* W, float* C, const int* start, const int* perm, int top, int E,
                             int rows, int N, int K, int lda, int ldc, hipStream_t st) {
  const int tiles = (rows / 64 + E) * ((N + 63) / 64);       // at least one part tile per group
  hipLaunchKernelGGL(gemm_f32_kernel<true>, dim3(tiles), dim3(256), 0, st, A, W, C, rows, N, K, lda, K, ldc,
                     GroupArgs{start, perm, top, E});
}

}  // namespace evgpt
