// The part of a decode step between a mixer's input projection and its output projection, for one token per
// sequence, in one launch: attention heads (norm, rotation, cache append), the matrix memory and the
// state-space recurrence with its convolution.  Inputs are the projection's fp32 rows or split-K slabs;
// what a prompt would have stored in T is rounded to T here as well.
//
// A recurrent state is streamed once: sixteen lanes per state row read it, decay it, add the token, dot it with
// the query and write it back.  A block owns some rows of one head; it prepares the head's small vectors
// (query, key, convolution outputs, gates) itself in LDS rather than waiting for another launch.
#include "src_rows.h"

namespace evgpt {

// rows of S (of one head) from v0 on, vb of them: S = decay S + add v k^T, y = S q
template <typename Y>
__device__ __forceinline__ void stream_state(float* __restrict__ S, int N, int v0, int vb, bool fresh, float decay,
                                             const float* qs, const float* ks, const float* avs, Y&& put) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l16 = lane & 15, rg = lane >> 4;
  for (int i = wid * 4 + rg; i < vb; i += 16) {
    float* Sr = S + static_cast<long long>(v0 + i) * N;
    const float av = avs[i];
    float y = 0.f;
    for (int e = l16 * 4; e < N; e += 64) {
      const f32x4_t kk = *reinterpret_cast<const f32x4_t*>(ks + e), qq = *reinterpret_cast<const f32x4_t*>(qs + e);
      f32x4_t s = kk * av;
      if (!fresh) s += load4(Sr + e) * decay;
      *reinterpret_cast<f32x4_t*>(Sr + e) = s;
#pragma unroll
      for (int j = 0; j < 4; ++j) y += s[j] * qq[j];
    }
    y = group_sum<16>(y);
    if (l16 == 0) put(i, y);
  }
}

template <typename T>
__device__ void head_step(const AttnPrepArgs& a, int b, int head, int p, bool live, float* red) {
  const bool is_q = head < a.Hq;
  const int h = is_q ? head : head - a.Hq;
  const int col = is_q ? a.q_col : a.k_col, width = (is_q ? a.Hq : a.Hkv) * a.D;
  const float* w = is_q ? a.qw : a.kw;
  float r = 1.f;
  if (w) {
    float s = 0.f;
    for (int c = threadIdx.x * 8; c < width; c += 2048) {
      float t[8];
      src8(a.src, b, col + c, t);
      s += sumsq8(t);
    }
    r = rsqrtf(block_sum(s, red) / static_cast<float>(is_q ? a.nq : a.nk) + a.eps);
  }
  if (!is_q && !live) return;
  const int half = a.rot >> 1, pt = min(max(p, 0), a.max_pos - 1);
  const float* cs = a.cos_tab + static_cast<long long>(pt) * half;
  const float* sn = a.sin_tab + static_cast<long long>(pt) * half;
  for (int d = threadIdx.x; d < a.D; d += 256) {
    const int c = h * a.D + d;
    float u = src1(a.src, b, col + c) * r;
    if (w) u *= w[c];
    if (d < a.rot) {
      const int i = d < half ? d : d - half, c2 = d < half ? c + half : c - half;
      float o = src1(a.src, b, col + c2) * r;
      if (w) o *= w[c2];
      u = d < half ? u * cs[i] - o * sn[i] : u * cs[i] + o * sn[i];
    }
    if (is_q) {
      static_cast<T*>(a.q_out)[static_cast<long long>(b) * width + c] = from_f32<T>(u);
    } else {
      const long long o = ((static_cast<long long>(b) * a.Hkv + h) * a.cap + max(p, 0) % a.cap) * a.D + d;
      static_cast<T*>(a.k_cache)[o] = from_f32<T>(u);
      static_cast<T*>(a.v_cache)[o] = from_f32<T>(src1(a.src, b, a.v_col + c));
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void parallel_step_kernel(StepHeads sh, StepMemory m, const int* __restrict__ pos,
                                                            const int* __restrict__ live, int vb) {
  extern __shared__ __attribute__((aligned(16))) float lds[];      // [N] query, [N] key, [vb] weighted values
  __shared__ float red[16], gates[2];
  const int b = blockIdx.y, p = pos[b];
  const bool alive = live == nullptr || live[b] != 0;
  const int n_heads = sh.on ? sh.a.Hq + sh.a.Hkv : 0;
  if (static_cast<int>(blockIdx.x) < n_heads) {
    head_step<T>(sh.a, b, blockIdx.x, p, alive, red);
    return;
  }
  const int per = m.V / vb, i0 = blockIdx.x - n_heads, h = i0 / per, v0 = (i0 % per) * vb;
  const int gi = b * m.H + h;
  if (!alive) {                         // a parked sequence keeps its state
    for (int i = threadIdx.x; i < vb; i += 256) m.out[static_cast<long long>(gi) * m.V + v0 + i] = 0.f;
    return;
  }
  const bool fresh = p <= 0;
  float *qs = lds, *ks = lds + m.N, *avs = ks + m.N;
  const long long from = (static_cast<long long>(p & 1) * m.slots + b) * m.H + h;
  const long long to = (static_cast<long long>((p + 1) & 1) * m.slots + b) * m.H + h;
  if (threadIdx.x == 0) {
    gates[0] = m.cap * tanhf((src1(m.src, b, m.i_col + h) + m.ib[h]) / m.cap);
    gates[1] = -softplus_f(-m.cap * tanhf((src1(m.src, b, m.f_col + h) + m.fb[h]) / m.cap));
  }
  for (int e = threadIdx.x; e < m.N; e += 256) {
    qs[e] = src_t<T>(m.src, b, m.q_col + h * m.N + e) * m.qscale;
    ks[e] = src_t<T>(m.src, b, m.k_col + h * m.N + e);
  }
  __syncthreads();
  const float m0 = fresh ? 0.f : m.m[from];
  const float li = gates[0], lf = gates[1], m1 = fmaxf(lf + m0, li);
  const float decay = expf(lf + m0 - m1), add = expf(li - m1);
  for (int i = threadIdx.x; i < vb; i += 256) avs[i] = add * src_t<T>(m.src, b, m.v_col + h * m.V + v0 + i);
  float dot = 0.f;
  for (int e = threadIdx.x; e < m.N; e += 256) {
    const float n1 = (fresh ? 0.f : m.n[from * m.N + e] * decay) + add * ks[e];
    if (v0 == 0) m.n[to * m.N + e] = n1;
    dot += n1 * qs[e];
  }
  dot = block_sum(dot, red);            // (its barriers also publish avs)
  if (v0 == 0 && threadIdx.x == 0) m.m[to] = m1;
  const float inv = 1.f / (fmaxf(fabsf(dot), expf(-m1)) + 1e-6f);
  float* out = m.out + static_cast<long long>(gi) * m.V + v0;
  stream_state(m.S + static_cast<long long>(gi) * m.V * m.N, m.N, v0, vb, fresh, decay, qs, ks, avs,
               [&](int i, float y) { out[i] = y * inv; });
}

template <typename T>
__global__ __launch_bounds__(256) void ssd_step_kernel(StepSsd a, const int* __restrict__ pos, const int* __restrict__ live,
                                                       int vb) {
  extern __shared__ __attribute__((aligned(16))) float lds[];      // [N] C, [N] B, [vb] weighted x, [vb] x
  __shared__ float gates[2];
  const int b = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * vb, p = pos[b];
  const int gi = b * a.H + h, per_group = a.H / a.G, g = h / per_group;
  float* out = a.out + static_cast<long long>(gi) * a.V + v0;
  if (live && !live[b]) {
    for (int i = threadIdx.x; i < vb; i += 256) out[i] = 0.f;
    return;
  }
  const bool fresh = p <= 0;
  float *cs = lds, *bs = lds + a.N, *avs = bs + a.N, *xs = avs + vb;
  const int C = a.H * a.V + 2 * a.G * a.N;
  if (threadIdx.x == 0) {
    const float dt = softplus_f(src1(a.src, b, a.dt_col + h) + a.dt_bias[h]);
    gates[0] = expf(-expf(a.a_log[h]) * dt);
    gates[1] = dt;
  }
  T* ring = static_cast<T*>(a.ring) + static_cast<long long>(b) * a.taps * C;
  for (int i = threadIdx.x; i < 2 * a.N + vb; i += 256) {
    const bool is_x = i >= 2 * a.N;
    const int c = is_x ? h * a.V + v0 + i - 2 * a.N
                       : a.H * a.V + (i < a.N ? g * a.N + i : (a.G + g) * a.N + i - a.N);     // B, then C
    const T cur = from_f32<T>(src1(a.src, b, a.x_col + c));
    float acc = a.conv_b[c];
    const float* w = a.conv_w + static_cast<long long>(c) * a.taps;
    for (int j = 0; j < a.taps; ++j) {
      const int d = a.taps - 1 - j;
      if (p - d < 0) continue;
      acc += w[j] * (d == 0 ? to_f32(cur) : to_f32(ring[static_cast<long long>((p - d) % a.taps) * C + c]));
    }
    const float v = to_f32(from_f32<T>(acc * sigmoid_f(acc)));
    if (is_x) xs[i - 2 * a.N] = v;
    else if (i < a.N) bs[i] = v;
    else cs[i - a.N] = v;
    // the current input's slot is read by nobody in this step; one block per channel stores it
    if (is_x || (v0 == 0 && h % per_group == 0)) ring[static_cast<long long>(max(p, 0) % a.taps) * C + c] = cur;
  }
  __syncthreads();
  const float decay = gates[0], dt = gates[1];
  for (int i = threadIdx.x; i < vb; i += 256) avs[i] = dt * xs[i];
  __syncthreads();
  const float skip = a.skip[h];
  stream_state(a.S + static_cast<long long>(gi) * a.V * a.N, a.N, v0, vb, fresh, decay, cs, bs, avs, [&](int i, float y) {
    const float z = src_t<T>(a.src, b, a.z_col + h * a.V + v0 + i);
    out[i] = (y + skip * xs[i]) * z * sigmoid_f(z);
  });
}

// state rows per block: sixteen keep a single stream's launch wide, more amortise the head's small vectors
static int rows_per_block(int heads, int V, int B) {
  int vb = 16;
  while (vb < 64 && V % (vb * 2) == 0 && static_cast<long long>(heads) * (V / vb) * B > 2048) vb *= 2;
  return vb;
}

void launch_parallel_step(const StepHeads& h, const StepMemory& m, const int* pos, const int* live, bool f32, int B,
                          hipStream_t st) {
  const int vb = rows_per_block(m.H, m.V, B);
  const dim3 grid((h.on ? h.a.Hq + h.a.Hkv : 0) + m.H * (m.V / vb), B);
  const size_t lds = (2 * m.N + vb) * 4;
  if (f32) hipLaunchKernelGGL(parallel_step_kernel<float>, grid, dim3(256), lds, st, h, m, pos, live, vb);
  else hipLaunchKernelGGL(parallel_step_kernel<bf16_t>, grid, dim3(256), lds, st, h, m, pos, live, vb);
}
void launch_ssd_step(const StepSsd& a, const int* pos, const int* live, bool f32, int B, hipStream_t st) {
  const int vb = rows_per_block(a.H, a.V, B);
  const dim3 grid(a.V / vb, a.H, B);
  const size_t lds = (2 * a.N + 2 * vb) * 4;
  if (f32) hipLaunchKernelGGL(ssd_step_kernel<float>, grid, dim3(256), lds, st, a, pos, live, vb);
  else hipLaunchKernelGGL(ssd_step_kernel<bf16_t>, grid, dim3(256), lds, st, a, pos, live, vb);
}

}  // namespace evgpt
