// Mixture of experts: routing, sorting of a prompt's tokens by expert, and the two products of a decode step of a
// few rows.  The grouped matrix products of a prompt are instances of gemm.hip (bf16) and gemm_f32.hip.
//
// Routing is fp32: the `top` largest of logits + bias, the lower index of equals first, softmax over the chosen.
// A decode step reads only the chosen experts' weights: every workgroup routes its row again from the logits (a few
// dozen numbers) and its waves stream units of four weight rows.
#include "src_rows.h"

namespace evgpt {

// One wave: z [E] in LDS is used up (a lane touches its own entries only); lane k < top returns its expert and weight.
__device__ __forceinline__ void route_row(const MoeRoute& a, long long row, float* z, int lane, int& expert, float& weight) {
  for (int e = lane; e < a.E; e += 64) z[e] = fmaxf(src1(a.z, row, e) + a.bias[e], -3.4e38f);   // (NaN: last)
  float best0 = 0.f, mine = -INFINITY;
  expert = 0;
  for (int k = 0; k < a.top; ++k) {
    float bv = -INFINITY;
    int be = 0x7fffffff;
    for (int e = lane; e < a.E; e += 64) {
      const float v = z[e];
      if (v > bv) { bv = v; be = e; }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(bv, off, 64);
      const int oe = __shfl_xor(be, off, 64);
      if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; }
    }
    be = min(be, a.E - 1);
    if (k == 0) best0 = bv;
    if (lane == k) { mine = bv; expert = be; }
    if ((be & 63) == lane) z[be] = -INFINITY;
  }
  const float e = lane < a.top ? expf(mine - best0) : 0.f;
  weight = e / wave_sum(e);
}

__global__ __launch_bounds__(256) void moe_route_kernel(MoeRoute a, int* __restrict__ idx, float* __restrict__ w, int rows) {
  extern __shared__ float z[];                     // [4][E]
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const long long row = blockIdx.x * 4ll + wid;
  if (row >= rows) return;
  int e;
  float f;
  route_row(a, row, z + wid * a.E, lane, e, f);
  if (lane < a.top) {
    idx[row * a.top + lane] = e;
    w[row * a.top + lane] = f;
  }
}
void launch_moe_route(const MoeRoute& r, int* idx, float* w, int rows, hipStream_t st) {
  hipLaunchKernelGGL(moe_route_kernel, dim3((rows + 3) / 4), dim3(256), 16 * r.E, st, r, idx, w, rows);
}

// Block e: the entries of expert e in order.  A thread owns a run of entries; its place is the count of matches before
// it, the expert's place the count of entries of earlier experts.
__global__ __launch_bounds__(1024) void moe_group_kernel(const int* __restrict__ idx, int* __restrict__ perm,
                                                         int* __restrict__ inv, int* __restrict__ start, int n, int E) {
  __shared__ int wave_n[16], wave_less[16];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int run = ((n + 1023) / 1024 + 3) / 4 * 4;           // whole vectors of four
  const int a = min(tid * run, n), b = min(a + run, n);
  int mine = 0, less = 0;
  for (int i = a; i < b; i += 4) {
    int v[4];
    if (i + 4 <= n) *reinterpret_cast<int4*>(v) = *reinterpret_cast<const int4*>(idx + i);
    else
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = idx[min(i + j, n - 1)];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (i + j < b) { mine += v[j] == e; less += v[j] < e; }
  }
  int before = mine, total_less = less;                      // inclusive scan and sum of the wave
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const int t = __shfl_up(before, off, 64);
    if (lane >= off) before += t;
    total_less += __shfl_xor(total_less, off, 64);
  }
  if (lane == 63) { wave_n[wid] = before; wave_less[wid] = total_less; }
  __syncthreads();
  int first = 0;
  for (int w = 0; w < 16; ++w) {
    first += wave_less[w];
    if (w < wid) before += wave_n[w];
  }
  int at = first + before - mine;
  for (int i = a; i < b; ++i)
    if (idx[i] == e) {
      perm[at] = i;
      inv[i] = at++;
    }
  if (tid == 0) {
    start[e] = first;
    if (e == E - 1) start[E] = n;
  }
}
void launch_moe_group(const int* idx, int* perm, int* inv, int* start, int n, int E, hipStream_t st) {
  hipLaunchKernelGGL(moe_group_kernel, dim3(E), dim3(1024), 0, st, idx, perm, inv, start, n, E);
}

__device__ __forceinline__ float dot_chunk(const u32x4_t& w, const u32x4_t& x, float acc, bf16_t) { return dot8_bf16(w, x, acc); }
__device__ __forceinline__ float dot_chunk(const u32x4_t& w, const u32x4_t& x, float acc, float) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc += __uint_as_float(w[i]) * __uint_as_float(x[i]);
  return acc;
}
// R weight rows times one input row of K elements by a wave; four 1 KB pieces of every row in flight
template <typename T, int R>
__device__ __forceinline__ void stream_rows(const T* const (&w)[R], const T* x, int K, int lane, float (&acc)[R]) {
  constexpr int CE = 16 / sizeof(T), U = 4;
  const int n = K / CE;
  for (int c0 = 0; c0 < n; c0 += 64 * U) {
    u32x4_t wv[U][R];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * 64 + lane;
      if (c < n)
#pragma unroll
        for (int r = 0; r < R; ++r) wv[u][r] = load_stream16(w[r] + static_cast<long long>(c) * CE);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + u * 64 + lane;
      if (c < n) {
        const u32x4_t xv = load16(x + static_cast<long long>(c) * CE);
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = dot_chunk(wv[u][r], xv, acc[r], T(0));
      }
    }
  }
}

// a row's experts and weights for the whole block
template <int TOP_MAX>
__device__ __forceinline__ void block_route(const MoeRoute& a, int b, float* z, int* sel, float* wsel) {
  const int lane = threadIdx.x & 63;
  if (threadIdx.x < 64) {
    int e;
    float f;
    route_row(a, b, z, lane, e, f);
    if (lane < a.top && lane < TOP_MAX) { sel[lane] = e; wsel[lane] = f; }
  }
  __syncthreads();
}

template <typename T>
__global__ __launch_bounds__(256) void moe_step_up_kernel(MoeStep a) {
  extern __shared__ float z[];                     // [E]
  __shared__ int sel[64];
  __shared__ float wsel[64];
  const int b = blockIdx.y, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  block_route<64>(a.route, b, z, sel, wsel);
  const T* x = static_cast<const T*>(a.x) + static_cast<long long>(b) * a.K;
  const int half = a.F / 2, units = a.route.top * half;
  for (int u = blockIdx.x * 4 + wid; u < units; u += gridDim.x * 4) {
    const int k = u / half, f = (u % half) * 2;
    const T* g = static_cast<const T*>(a.w) + (static_cast<long long>(sel[k]) * 2 * a.F + f) * a.K;
    const T* up = g + static_cast<long long>(a.F) * a.K;
    const T* const rows[4] = {g, g + a.K, up, up + a.K};
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    stream_rows<T, 4>(rows, x, a.K, lane, acc);
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] = wave_sum(acc[r]);
    if (lane < 2) {
      const float gt = lane ? acc[1] : acc[0], uv = lane ? acc[3] : acc[2];
      static_cast<T*>(a.h)[(static_cast<long long>(b) * a.route.top + k) * a.F + f + lane] =
          from_f32<T>((a.act == GLU_SILU ? gt * sigmoid_f(gt) : gelu_tanh_f(gt)) * uv);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void moe_step_down_kernel(MoeStep a) {
  extern __shared__ float z[];                     // [E]
  __shared__ int sel[64];
  __shared__ float wsel[64];
  const int b = blockIdx.y, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  block_route<64>(a.route, b, z, sel, wsel);
  const int units = a.N / 2;
  for (int u = blockIdx.x * 4 + wid; u < units; u += gridDim.x * 4) {
    float s0 = 0.f, s1 = 0.f;
    for (int k = 0; k < a.route.top; ++k) {
      const T* w = static_cast<const T*>(a.w) + (static_cast<long long>(sel[k]) * a.N + u * 2) * a.F;
      const T* const rows[2] = {w, w + a.F};
      float acc[2] = {0.f, 0.f};
      stream_rows<T, 2>(rows, static_cast<const T*>(a.x) + (static_cast<long long>(b) * a.route.top + k) * a.F, a.F, lane, acc);
      s0 += wsel[k] * acc[0];
      s1 += wsel[k] * acc[1];
    }
    s0 = wave_sum(s0);
    s1 = wave_sum(s1);
    if (lane < 2) a.y[static_cast<long long>(b) * a.N + u * 2 + lane] = lane ? s1 : s0;
  }
}
static int step_blocks(int units) {
  const int want = (units + 3) / 4;
  return want < 1024 ? want : 1024;
}
void launch_moe_step_up(const MoeStep& a, bool f32, int B, hipStream_t st) {
  const dim3 grid(step_blocks(a.route.top * (a.F / 2)), B), block(256);
  if (f32) hipLaunchKernelGGL(moe_step_up_kernel<float>, grid, block, 4 * a.route.E, st, a);
  else hipLaunchKernelGGL(moe_step_up_kernel<bf16_t>, grid, block, 4 * a.route.E, st, a);
}
void launch_moe_step_down(const MoeStep& a, bool f32, int B, hipStream_t st) {
  const dim3 grid(step_blocks(a.N / 2), B), block(256);
  if (f32) hipLaunchKernelGGL(moe_step_down_kernel<float>, grid, block, 4 * a.route.E, st, a);
  else hipLaunchKernelGGL(moe_step_down_kernel<bf16_t>, grid, block, 4 * a.route.E, st, a);
}

}  // namespace evgpt
