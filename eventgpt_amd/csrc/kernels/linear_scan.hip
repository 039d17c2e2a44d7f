// Linear recurrences with one scalar decay per head and token (Mamba-2's state-space duality, the matrix
// memory of xLSTM):
//     S_t = exp(a_t) S_(t-1) + b_t v_t k_t^T,      y_t = S_t q_t          (S is [V][N], value-major)
//
// Prefill runs in chunks of 64 tokens, three launches, all chunks of all sequences at once where the
// recurrence allows it.  With F_t = sum of a over the chunk up to t:
//   1. scan_chunk_state: what a chunk adds to the state,  dS = sum_s exp(F_L - F_s) b_s v_s k_s^T;
//   2. scan_chunk_pass: the walk over a sequence's chunks, elementwise:  S <- exp(F_L) S + dS; every
//      chunk's slot of dS ends up holding the state at the chunk's START;
//   3. scan_chunk_out: y_t = exp(F_t) S_start q_t + sum_{s <= t} exp(F_t - F_s) b_s (q_t . k_s) v_s.
// The products run on MFMA.  Whatever belongs to the recurrence -- states, decays, weighted scores --
// stays fp32: decay sums are accumulated in double (differences of long sums are taken), and fp32 MFMA
// operands go in as two bf16 parts (`WideFrag`).
//
// With a running maximum (log_in given; b = exp(log_in)) the stored state is S exp(-m), with
// m_t = max(a_t + m_(t-1), log_in_t), and a normaliser n_t (the same recurrence on k alone) divides the
// output: y_t = S_t q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).  m is a max-plus scan, so it chunks too:
// m_t = F_t + max(m_start, max_{s <= t}(log_in_s - F_s)).
//
// Decode (scan_step) streams the state once: sixteen lanes per state row, read, decayed, updated, dotted
// with q and written back in one pass.
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

constexpr int SL = SCAN_CHUNK;
constexpr int TS = SL + 8;      // elements per row of a transposed LDS tile

// inclusive sum over the wave, in double
__device__ __forceinline__ double wave_scan_add(double v) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const double o = __shfl_up(v, d, 64);
    if (lane >= d) v += o;
  }
  return v;
}
__device__ __forceinline__ float wave_scan_max(float v) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const float o = __shfl_up(v, d, 64);
    if (lane >= d) v = fmaxf(v, o);
  }
  return v;
}

// rows [row0, row0 + len) x 64 columns from col (nc of them exist) of a T matrix, transposed into
// lds[column][row] with rows past len as zeros
template <typename T>
__device__ __forceinline__ void load_transposed(const T* __restrict__ p, long long ld, long long row0, int len, int col,
                                                int nc, T* lds) {
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int idx = threadIdx.x + i * 256, s = idx & 63, c8 = (idx >> 6) * 8;
    T t[8];
    if (s < len && c8 < nc) {
      const T* g = p + (row0 + s) * ld + col + c8;
      if constexpr (sizeof(T) == 2) *reinterpret_cast<u32x4_t*>(t) = load16(g);
      else {
        *reinterpret_cast<f32x4_t*>(t) = load4(g);
        *reinterpret_cast<f32x4_t*>(t + 4) = load4(g + 4);
      }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) t[j] = T(0);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) lds[(c8 + j) * TS + s] = t[j];
  }
}

template <typename T, bool STAB>
__global__ __launch_bounds__(256) void scan_chunk_state_kernel(ScanArgs a, ScanChunks c) {
  __shared__ __attribute__((aligned(16))) T kt[64 * TS];
  __shared__ __attribute__((aligned(16))) T vt[64 * TS];
  __shared__ __attribute__((aligned(16))) float wgt[SL];
  const int nt = (a.N + 63) >> 6;
  const int n0 = (blockIdx.x % nt) * 64, v0 = (blockIdx.x / nt) * 64;
  const int h = blockIdx.y, ci = blockIdx.z;
  const int row0 = c.chunks[ci * 4], len = min(c.chunks[ci * 4 + 1], SL);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int nn = min(64, a.N - n0), nv = min(64, a.V - v0);
  load_transposed(static_cast<const T*>(a.k), a.ldk, row0, len, (h / a.per_group) * a.N + n0, nn, kt);
  load_transposed(static_cast<const T*>(a.v), a.ldv, row0, len, h * a.V + v0, nv, vt);
  if (wid == 0) {
    const bool in = lane < len;
    const long long gi = static_cast<long long>(row0 + lane) * a.H + h;
    const double F = wave_scan_add(in ? static_cast<double>(a.log_decay[gi]) : 0.0);
    const double FL = __shfl(F, 63, 64);
    float e = static_cast<float>(FL - F), top = 0.f, b = 1.f;
    if constexpr (STAB) {
      e = in ? e + a.log_in[gi] : -INFINITY;
      top = wave_max(e);
    } else {
      b = in ? a.scale_in[gi] : 0.f;
    }
    wgt[lane] = in ? expf(e - top) * b : 0.f;
    if (blockIdx.x == 0 && lane == 0) {
      const long long o = static_cast<long long>(ci) * a.H + h;
      c.am[o] = top;
      c.fl[o] = static_cast<float>(FL);
    }
  }
  __syncthreads();
  // D[v][n]: a wave owns 16 value rows
  f32x4_t acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ks = 0; ks < SL / 32; ++ks) {
    float x[8], w[8];
    load8(vt + (wid * 16 + fr) * TS + ks * 32 + g * 8, x);
    load8(wgt + ks * 32 + g * 8, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= w[j];
    const WideFrag<T> vf = wide_frag<T>(x);
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = mma(vf, load_frag(kt + (i * 16 + fr) * TS + ks * 32 + g * 8), acc[i]);
  }
  float* dS = c.dS + (static_cast<long long>(ci) * a.H + h) * a.V * a.N;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int v = wid * 16 + g * 4 + r, n = i * 16 + fr;
      if (v < nv && n < nn) dS[static_cast<long long>(v0 + v) * a.N + n0 + n] = acc[i][r];
    }
  if constexpr (STAB) {
    if (v0 == 0 && tid < nn) {
      float s = 0.f;
      for (int t = 0; t < SL; ++t) s += wgt[t] * to_f32(kt[tid * TS + t]);
      c.dn[(static_cast<long long>(ci) * a.H + h) * a.N + n0 + tid] = s;
    }
  }
}

// One thread per four state elements (the block after the last: the normaliser), over a sequence's chunks.
template <bool STAB>
__global__ __launch_bounds__(256) void scan_chunk_pass_kernel(ScanArgs a, ScanChunks c) {
  const int* sq = c.seqs + blockIdx.z * 4;
  const int c0 = sq[0], nc = sq[1];
  const long long slot = sq[2];
  const bool fresh = sq[3] != 0;
  const int h = blockIdx.y;
  const long long per = static_cast<long long>(a.V) * a.N;
  const bool norm = STAB && blockIdx.x == gridDim.x - 1;
  const long long size = norm ? a.N : per;
  const long long e0 = norm ? threadIdx.x * 4ll : (static_cast<long long>(blockIdx.x) * 256 + threadIdx.x) * 4;
  const float m_in = STAB && !fresh ? a.m[slot * a.H + h] : 0.f;
  float* state = norm ? a.n + (slot * a.H + h) * a.N : a.S + (slot * a.H + h) * per;
  float* dbase = norm ? c.dn : c.dS;
  const bool lead = blockIdx.x == 0 && threadIdx.x == 0;
  for (long long e = e0; e < size; e += norm ? 1024 : size) {
    f32x4_t s = fresh ? f32x4_t{0.f, 0.f, 0.f, 0.f} : load4(state + e);
    float m = m_in;
    constexpr int PF = 4;            // chunk slots in flight
    f32x4_t nxt[PF];
#pragma unroll
    for (int k = 0; k < PF; ++k)
      if (k < nc) nxt[k] = load4(dbase + (static_cast<long long>(c0 + k) * a.H + h) * size + e);
    for (int k0 = 0; k0 < nc; k0 += PF) {
#pragma unroll
      for (int k = 0; k < PF; ++k) {
        if (k0 + k >= nc) break;
        const long long o = static_cast<long long>(c0 + k0 + k) * a.H + h;
        const f32x4_t d = nxt[k];
        if (k0 + k + PF < nc) nxt[k] = load4(dbase + (o + static_cast<long long>(PF) * a.H) * size + e);
        *reinterpret_cast<f32x4_t*>(dbase + o * size + e) = s;
        const float fl = c.fl[o];
        if constexpr (STAB) {
          const float am = c.am[o];
          if (lead) c.m0[o] = m;
          const float m1 = fmaxf(fl + m, am);
          const float x = expf(fl + m - m1), y = expf(am - m1);
          s = s * x + d * y;
          m = m1;
        } else {
          s = s * expf(fl) + d;
        }
      }
    }
    *reinterpret_cast<f32x4_t*>(state + e) = s;
  }
}

template <typename T, bool STAB>
__global__ __launch_bounds__(256) void scan_chunk_out_kernel(ScanArgs a, ScanChunks c) {
  __shared__ __attribute__((aligned(16))) T vt[64 * TS];
  __shared__ double F_s[SL];
  __shared__ float in_s[SL], m_s[SL], b_s[SL];
  const int v0 = blockIdx.x * 64, h = blockIdx.y, ci = blockIdx.z;
  const int row0 = c.chunks[ci * 4], len = min(c.chunks[ci * 4 + 1], SL);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int nv = min(64, a.V - v0), hk = h / a.per_group;
  const long long ho = static_cast<long long>(ci) * a.H + h;
  load_transposed(static_cast<const T*>(a.v), a.ldv, row0, len, h * a.V + v0, nv, vt);
  const float m0 = STAB ? c.m0[ho] : 0.f;
  if (wid == 0) {
    const bool in = lane < len;
    const long long gi = static_cast<long long>(row0 + lane) * a.H + h;
    const double F = wave_scan_add(in ? static_cast<double>(a.log_decay[gi]) : 0.0);
    F_s[lane] = F;
    if constexpr (STAB) {
      const float li = in ? a.log_in[gi] : -INFINITY;
      in_s[lane] = li;
      const float top = fmaxf(m0, wave_scan_max(static_cast<float>(static_cast<double>(li) - F)));
      const float m = static_cast<float>(F + static_cast<double>(top));
      m_s[lane] = m;
      if (blockIdx.x == 0 && lane == len - 1 && c.chunks[ci * 4 + 3])
        a.m[static_cast<long long>(c.chunks[ci * 4 + 2]) * a.H + h] = fmaxf(c.fl[ho] + m0, c.am[ho]);
    } else {
      b_s[lane] = in ? a.scale_in[gi] : 0.f;
    }
  }
  __syncthreads();
  if (wid * 16 >= len) return;
  // lane: token t of this wave's sixteen
  const int t = wid * 16 + fr, tc = min(t, len - 1);
  const T* qp = static_cast<const T*>(a.q) + (row0 + tc) * a.ldq + static_cast<long long>(hk) * a.N;
  const T* kp = static_cast<const T*>(a.k) + static_cast<long long>(hk) * a.N;
  const float* S0 = c.dS + ho * a.V * a.N + static_cast<long long>(v0) * a.N;
  const float* nrm = STAB ? c.dn + ho * a.N : nullptr;
  f32x4_t st[4], inter[4], y[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) st[i] = inter[i] = y[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float nq = 0.f;
  for (int n = g * 8; n < a.N; n += 32) {
    const Frag<T> qf = load_frag(qp + n);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i <= wid) {
        const int s = min(i * 16 + fr, len - 1);
        st[i] = mma(load_frag(kp + (row0 + s) * a.ldk + n), qf, st[i]);
      }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i * 16 < nv) {
        float x[8];
        load8(S0 + static_cast<long long>(i * 16 + fr) * a.N + n, x);
        inter[i] = mma(wide_frag<T>(x), qf, inter[i]);
      }
    if constexpr (STAB) {
      float x[8], q8[8];
      load8(nrm + n, x);
      load8(qp + n, q8);
#pragma unroll
      for (int j = 0; j < 8; ++j) nq += x[j] * q8[j];
    }
  }
  // weighted scores of this lane's token; the accumulator layout is the operand layout of the next product
  // with contraction slot (g, j) <-> key 32 b + 4 g + j (j < 4) or 32 b + 16 + 4 g + j - 4
  const double Ft = F_s[tc];
  const float mt = STAB ? m_s[tc] : 0.f;
  float den = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = i * 16 + g * 4 + r;
      float w = 0.f;
      if (s <= t && s < len) {
        w = static_cast<float>(Ft - F_s[s]);
        if constexpr (STAB) w = expf(w + in_s[s] - mt);
        else w = expf(w) * b_s[s];
      }
      st[i][r] *= w * a.qscale;
      den += st[i][r];
    }
#pragma unroll
  for (int kb = 0; kb < 2; ++kb) {
    if (kb * 2 > wid) break;
    float x[8];
#pragma unroll
    for (int j = 0; j < 4; ++j) { x[j] = st[kb * 2][j]; x[4 + j] = st[kb * 2 + 1][j]; }
    const WideFrag<T> pf = wide_frag<T>(x);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i * 16 < nv) {
        const T* vr = vt + (i * 16 + fr) * TS + kb * 32 + g * 4;
        Frag<T> vf;
        if constexpr (sizeof(T) == 2) {
          const u32x2_t lo = *reinterpret_cast<const u32x2_t*>(vr), hi = *reinterpret_cast<const u32x2_t*>(vr + 16);
          vf.v = __builtin_bit_cast(bf16x8_t, u32x4_t{lo[0], lo[1], hi[0], hi[1]});
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) { vf.v[j] = vr[j]; vf.v[4 + j] = vr[16 + j]; }
        }
        y[i] = mma(vf, pf, y[i]);
      }
  }
  const float carry = expf(static_cast<float>(Ft + static_cast<double>(m0)) - mt) * a.qscale;
  float inv = 1.f;
  if constexpr (STAB) {
    den += __shfl_xor(den, 16, 64);
    den += __shfl_xor(den, 32, 64);
    nq += __shfl_xor(nq, 16, 64);
    nq += __shfl_xor(nq, 32, 64);
    inv = 1.f / (fmaxf(fabsf(nq * carry + den), expf(-mt)) + 1e-6f);
  }
  if (t >= len) return;
  const float skip = a.skip ? a.skip[h] : 0.f;
  T* o = static_cast<T*>(a.out) + (static_cast<long long>(row0 + t) * a.H + h) * a.V + v0;
  const T* vrow = static_cast<const T*>(a.v) + (row0 + t) * a.ldv + static_cast<long long>(h) * a.V + v0;
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (i * 16 < nv) {
      const int v = i * 16 + g * 4;
      f32x4_t r = (inter[i] * carry + y[i]) * inv;
      if (a.skip) r += load4(vrow + v) * skip;
      store4(o + v, r[0], r[1], r[2], r[3]);
    }
}

void launch_scan_prefill(const ScanArgs& a, const ScanChunks& c, bool f32, hipStream_t st) {
  const int nt = (a.N + 63) / 64, vt = (a.V + 63) / 64;
  const bool stab = a.log_in != nullptr;
  const dim3 g1(nt * vt, a.H, c.C), g3(vt, a.H, c.C);
  const long long quads = static_cast<long long>(a.V) * a.N / 4;
  const dim3 g2(static_cast<unsigned>((quads + 255) / 256) + (stab ? 1 : 0), a.H, c.nseq);
  if (f32) {
    if (stab) hipLaunchKernelGGL((scan_chunk_state_kernel<float, true>), g1, dim3(256), 0, st, a, c);
    else hipLaunchKernelGGL((scan_chunk_state_kernel<float, false>), g1, dim3(256), 0, st, a, c);
  } else {
    if (stab) hipLaunchKernelGGL((scan_chunk_state_kernel<bf16_t, true>), g1, dim3(256), 0, st, a, c);
    else hipLaunchKernelGGL((scan_chunk_state_kernel<bf16_t, false>), g1, dim3(256), 0, st, a, c);
  }
  if (stab) hipLaunchKernelGGL(scan_chunk_pass_kernel<true>, g2, dim3(256), 0, st, a, c);
  else hipLaunchKernelGGL(scan_chunk_pass_kernel<false>, g2, dim3(256), 0, st, a, c);
  if (f32) {
    if (stab) hipLaunchKernelGGL((scan_chunk_out_kernel<float, true>), g3, dim3(256), 0, st, a, c);
    else hipLaunchKernelGGL((scan_chunk_out_kernel<float, false>), g3, dim3(256), 0, st, a, c);
  } else {
    if (stab) hipLaunchKernelGGL((scan_chunk_out_kernel<bf16_t, true>), g3, dim3(256), 0, st, a, c);
    else hipLaunchKernelGGL((scan_chunk_out_kernel<bf16_t, false>), g3, dim3(256), 0, st, a, c);
  }
}

// One token.  Block: sixteen state rows of one head; sixteen lanes per row.  Every block of a head computes
// the new maximum and the normaliser's dot product itself; the normaliser and the maximum are stored by a
// second launch, when all of them have read the old ones.
template <typename T, bool STAB>
__global__ __launch_bounds__(256) void scan_step_kernel(ScanArgs a, const int* __restrict__ pos,
                                                        const int* __restrict__ live) {
  const int h = blockIdx.y, b = blockIdx.z, v0 = blockIdx.x * 16;
  if (live && !live[b]) return;       // a parked sequence keeps its state
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l16 = lane & 15, rg = lane >> 4;
  const bool fresh = pos[b] <= 0;
  const int hk = h / a.per_group;
  const T* q = static_cast<const T*>(a.q) + b * a.ldq + static_cast<long long>(hk) * a.N;
  const T* k = static_cast<const T*>(a.k) + b * a.ldk + static_cast<long long>(hk) * a.N;
  const int gi = b * a.H + h;
  float decay, add, inv = 1.f;
  const int v = v0 + wid * 4 + rg;
  float* Sr = a.S + (static_cast<long long>(gi) * a.V + v) * a.N;
  if constexpr (STAB) {
    const float m = fresh ? 0.f : a.m[gi];
    const float lf = a.log_decay[gi], li = a.log_in[gi];
    const float m1 = fmaxf(lf + m, li);
    decay = expf(lf + m - m1);
    add = expf(li - m1);
    float dot = 0.f;
    const float* n = a.n + static_cast<long long>(gi) * a.N;
    for (int e = l16 * 4; e < a.N; e += 64) {
      const f32x4_t kk = load4(k + e), qq = load4(q + e);
      const f32x4_t nn = fresh ? kk * add : load4(n + e) * decay + kk * add;
#pragma unroll
      for (int i = 0; i < 4; ++i) dot += nn[i] * qq[i];
    }
    dot = group_sum<16>(dot) * a.qscale;
    inv = 1.f / (fmaxf(fabsf(dot), expf(-m1)) + 1e-6f);
  } else {
    decay = expf(a.log_decay[gi]);
    add = a.scale_in[gi];
  }
  const float vv = to_f32(static_cast<const T*>(a.v)[b * a.ldv + static_cast<long long>(h) * a.V + v]);
  const float av = add * vv;
  float y = 0.f;
  for (int e = l16 * 4; e < a.N; e += 64) {
    const f32x4_t kk = load4(k + e), qq = load4(q + e);
    f32x4_t s = kk * av;
    if (!fresh) s += load4(Sr + e) * decay;
    *reinterpret_cast<f32x4_t*>(Sr + e) = s;
#pragma unroll
    for (int i = 0; i < 4; ++i) y += s[i] * qq[i];
  }
  y = group_sum<16>(y) * a.qscale * inv;
  if (a.skip) y += a.skip[h] * vv;
  if (l16 == 0) static_cast<T*>(a.out)[(static_cast<long long>(b) * a.H + h) * a.V + v] = from_f32<T>(y);
}

// normaliser and maximum of the step, after every block of scan_step has read the old ones
template <typename T>
__global__ __launch_bounds__(256) void scan_step_norm_kernel(ScanArgs a, const int* __restrict__ pos,
                                                             const int* __restrict__ live) {
  const int h = blockIdx.x, b = blockIdx.y;
  if (live && !live[b]) return;
  const bool fresh = pos[b] <= 0;
  const int gi = b * a.H + h;
  const T* k = static_cast<const T*>(a.k) + b * a.ldk + static_cast<long long>(h / a.per_group) * a.N;
  const float m = fresh ? 0.f : a.m[gi];
  const float lf = a.log_decay[gi], li = a.log_in[gi];
  const float m1 = fmaxf(lf + m, li);
  const float decay = expf(lf + m - m1), add = expf(li - m1);
  float* n = a.n + static_cast<long long>(gi) * a.N;
  for (int e = threadIdx.x * 4; e < a.N; e += 1024) {
    f32x4_t nn = load4(k + e) * add;
    if (!fresh) nn += load4(n + e) * decay;
    *reinterpret_cast<f32x4_t*>(n + e) = nn;
  }
  __syncthreads();
  if (threadIdx.x == 0) a.m[gi] = m1;
}

void launch_scan_step(const ScanArgs& a, const int* pos, const int* live, bool f32, int B, hipStream_t st) {
  const dim3 grid(a.V / 16, a.H, B);
  const bool stab = a.log_in != nullptr;
  if (f32) {
    if (stab) {
      hipLaunchKernelGGL((scan_step_kernel<float, true>), grid, dim3(256), 0, st, a, pos, live);
      hipLaunchKernelGGL(scan_step_norm_kernel<float>, dim3(a.H, B), dim3(256), 0, st, a, pos, live);
    } else hipLaunchKernelGGL((scan_step_kernel<float, false>), grid, dim3(256), 0, st, a, pos, live);
  } else {
    if (stab) {
      hipLaunchKernelGGL((scan_step_kernel<bf16_t, true>), grid, dim3(256), 0, st, a, pos, live);
      hipLaunchKernelGGL(scan_step_norm_kernel<bf16_t>, dim3(a.H, B), dim3(256), 0, st, a, pos, live);
    } else hipLaunchKernelGGL((scan_step_kernel<bf16_t, false>), grid, dim3(256), 0, st, a, pos, live);
  }
}

}  // namespace evgpt
