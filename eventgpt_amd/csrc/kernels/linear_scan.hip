// Linear recurrences with one scalar decay per head and token (Mamba-2's state-space duality, the matrix
// memory of xLSTM):
//     S_t = exp(a_t) S_(t-1) + b_t v_t k_t^T,      y_t = S_t q_t          (S is [V][N], value-major)
//
// Prefill runs in chunks of 128 tokens (64 with fp32 storage), three launches, all chunks of all sequences at once where the
// recurrence allows it.  With F_t = sum of a over the chunk up to t:
//   1. scan_chunk_state: what a chunk adds to the state,  dS = sum_s exp(F_L - F_s) b_s v_s k_s^T;
//   2. scan_chunk_pass: the walk over a sequence's chunks, elementwise:  S <- exp(F_L) S + dS; every
//      chunk's slot of dS ends up holding the state at the chunk's START;
//   3. scan_chunk_out: y_t = exp(F_t) S_start q_t + sum_{s <= t} exp(F_t - F_s) b_s (q_t . k_s) v_s.
// The products run on MFMA.  Whatever belongs to the recurrence -- states, decays, weighted scores --
// stays fp32: decay sums and maxima are kept in double (differences of long sums are taken), and fp32 MFMA
// operands go in as two bf16 parts (`WideFrag`).
//
// With a running maximum (log_in given; b = exp(log_in)) the stored state is S exp(-m), with
// m_t = max(a_t + m_(t-1), log_in_t), and a normaliser n_t (the same recurrence on k alone) divides the
// output: y_t = S_t q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).  m is a max-plus scan, so it chunks too:
// m_t = F_t + max(m_start, max_{s <= t}(log_in_s - F_s)).
//
// n and m are stored twice, indexed by the parity of the position they are read at, so that a decode step
// (decode_step.hip) can write the next ones while other blocks still read the old ones.
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

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
__device__ __forceinline__ double wave_scan_max(double v) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const double o = __shfl_up(v, d, 64);
    if (lane >= d) v = fmax(v, o);
  }
  return v;
}
__device__ __forceinline__ double wave_max_f64(double v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v = fmax(v, __shfl_xor(v, off, 64));
  return v;
}

// rows [row0, row0 + len) x 64 columns from col (nc of them exist) of a T matrix, transposed into
// lds[column][row] with rows past len as zeros
template <typename T, int SL>
__device__ __forceinline__ void load_transposed(const T* __restrict__ p, long long ld, long long row0, int len, int col,
                                                int nc, T* lds) {
#pragma unroll
  for (int i = 0; i < SL / 32; ++i) {
    const int idx = threadIdx.x + i * 256, s = idx % SL, c8 = (idx / SL) * 8;
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
    for (int j = 0; j < 8; ++j) lds[(c8 + j) * (SL + 8) + s] = t[j];
  }
}

// One wave: decay sums F of a chunk's tokens (lane l: tokens l NH .. l NH + NH - 1), and with STAB the running maxima
// of log_in - F.
template <int NH, bool STAB>
__device__ __forceinline__ void chunk_gates(const ScanArgs& a, int row0, int len, int h, double (&F)[NH], float (&li)[NH],
                                            double (&top)[NH]) {
  const int lane = threadIdx.x & 63;
  double sum = 0.0;
#pragma unroll
  for (int i = 0; i < NH; ++i) {
    const int t = lane * NH + i;
    const long long gi = static_cast<long long>(row0 + t) * a.H + h;
    sum += t < len ? static_cast<double>(a.log_decay[gi]) : 0.0;
    F[i] = sum;
    if constexpr (STAB) li[i] = t < len ? a.log_in[gi] : -INFINITY;
    else li[i] = t < len ? a.scale_in[gi] : 0.f;
  }
  const double before = wave_scan_add(sum) - sum;
#pragma unroll
  for (int i = 0; i < NH; ++i) F[i] += before;
  if constexpr (STAB) {
    double m = -INFINITY;
#pragma unroll
    for (int i = 0; i < NH; ++i) {
      m = fmax(m, static_cast<double>(li[i]) - F[i]);
      top[i] = m;
    }
    const double up = __shfl_up(wave_scan_max(m), 1, 64);
    if (lane > 0)
#pragma unroll
      for (int i = 0; i < NH; ++i) top[i] = fmax(top[i], up);
  }
}

// Block: 64 value rows of one head and chunk, all of N in runs of 64.
template <typename T, bool STAB, int SL>
__global__ __launch_bounds__(256) void scan_chunk_state_kernel(ScanArgs a, ScanChunks c) {
  constexpr int TS = SL + 8, NH = SL / 64;
  __shared__ __attribute__((aligned(16))) T kt[64 * TS];
  __shared__ __attribute__((aligned(16))) T vt[64 * TS];
  __shared__ __attribute__((aligned(16))) float wgt[SL];
  const int v0 = blockIdx.x * 64, h = blockIdx.y, ci = blockIdx.z;
  const int row0 = c.chunks[ci * 4], len = min(c.chunks[ci * 4 + 1], SL);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int nv = min(64, a.V - v0), k_col = (h / a.per_group) * a.N;
  load_transposed<T, SL>(static_cast<const T*>(a.v), a.ldv, row0, len, h * a.V + v0, nv, vt);
  load_transposed<T, SL>(static_cast<const T*>(a.k), a.ldk, row0, len, k_col, min(64, a.N), kt);
  if (wid == 0) {
    double F[NH], m[NH];
    float li[NH];
    chunk_gates<NH, STAB>(a, row0, len, h, F, li, m);
    const double FL = __shfl(F[NH - 1], 63, 64);
    double top = 0.0;
    if constexpr (STAB) top = FL + __shfl(m[NH - 1], 63, 64);     // the largest FL - F + log_in
#pragma unroll
    for (int i = 0; i < NH; ++i) {
      const float e = static_cast<float>(FL - F[i] + (STAB ? static_cast<double>(li[i]) - top : 0.0));
      wgt[lane * NH + i] = lane * NH + i < len ? expf(e) * (STAB ? 1.f : li[i]) : 0.f;
    }
    if (blockIdx.x == 0 && lane == 0) {
      const long long o = static_cast<long long>(ci) * a.H + h;
      c.am[o] = top;
      c.fl[o] = FL;
    }
  }
  __syncthreads();
  WideFrag<T> vf[SL / 32];          // a wave owns 16 value rows, weighted
#pragma unroll
  for (int ks = 0; ks < SL / 32; ++ks) {
    float x[8], w[8];
    load8(vt + (wid * 16 + fr) * TS + ks * 32 + g * 8, x);
    load8(wgt + ks * 32 + g * 8, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= w[j];
    vf[ks] = wide_frag<T>(x);
  }
  float* dS = c.dS + ((static_cast<long long>(ci) * a.H + h) * a.V + v0) * a.N;
  for (int n0 = 0; n0 < a.N; n0 += 64) {
    const int nn = min(64, a.N - n0);
    if (n0 > 0) {
      __syncthreads();
      load_transposed<T, SL>(static_cast<const T*>(a.k), a.ldk, row0, len, k_col + n0, nn, kt);
      __syncthreads();
    }
    f32x4_t acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < SL / 32; ++ks)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = mma(load_frag(kt + (i * 16 + fr) * TS + ks * 32 + g * 8), vf[ks], acc[i]);
    // D[n][v]: a lane holds four consecutive n of value row fr
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int v = wid * 16 + fr, n = i * 16 + g * 4;
      if (v < nv && n < nn) *reinterpret_cast<f32x4_t*>(dS + static_cast<long long>(v) * a.N + n0 + n) = acc[i];
    }
    if constexpr (STAB) {
      if (v0 == 0 && tid < nn) {
        float s = 0.f;
        for (int t = 0; t < SL; ++t) s += wgt[t] * to_f32(kt[tid * TS + t]);
        c.dn[(static_cast<long long>(ci) * a.H + h) * a.N + n0 + tid] = s;
      }
    }
  }
}

// One thread per four state elements (the block after the last: the normaliser), over a sequence's chunks.
template <bool STAB>
__global__ __launch_bounds__(256) void scan_chunk_pass_kernel(ScanArgs a, ScanChunks c) {
  const int* sq = c.seqs + blockIdx.z * 4;
  const int c0 = sq[0], nc = sq[1];
  const long long slot = sq[2];
  const bool fresh = (sq[3] & 1) != 0;
  const long long nm_in = (static_cast<long long>(sq[3] >> 1 & 1) * a.slots + slot) * a.H;    // [2][slots][H]
  const long long nm_out = (static_cast<long long>(sq[3] >> 2 & 1) * a.slots + slot) * a.H;
  const int h = blockIdx.y;
  const long long per = static_cast<long long>(a.V) * a.N;
  const bool norm = STAB && blockIdx.x == gridDim.x - 1;
  const long long size = norm ? a.N : per;
  const long long e0 = norm ? threadIdx.x * 4ll : (static_cast<long long>(blockIdx.x) * 256 + threadIdx.x) * 4;
  const float m_in = STAB && !fresh ? a.m[nm_in + h] : 0.f;
  const float* from = norm ? a.n + (nm_in + h) * a.N : a.S + (slot * a.H + h) * per;
  float* to = norm ? a.n + (nm_out + h) * a.N : a.S + (slot * a.H + h) * per;
  float* dbase = norm ? c.dn : c.dS;
  const bool lead = blockIdx.x == 0 && threadIdx.x == 0;
  for (long long e = e0; e < size; e += norm ? 1024 : size) {
    f32x4_t s = fresh ? f32x4_t{0.f, 0.f, 0.f, 0.f} : load4(from + e);
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
        const double fl = c.fl[o];
        if constexpr (STAB) {
          const double am = c.am[o];
          if (lead) c.m0[o] = m;
          const float m1 = static_cast<float>(fmax(fl + m, am));
          const float x = expf(static_cast<float>(fl + m - m1)), y = expf(static_cast<float>(am - m1));
          s = s * x + d * y;
          m = m1;
        } else {
          s = s * expf(static_cast<float>(fl)) + d;
        }
      }
    }
    *reinterpret_cast<f32x4_t*>(to + e) = s;
  }
}

// Block: 64 value columns of one head and chunk.  Scores are computed transposed, a wave per sixteen keys of every
// 64, and meet in LDS (in the query tile's place); then a wave owns sixteen value rows for all tokens, so that the
// chunk's start state -- most of the bytes this kernel reads -- is read once.
template <typename T, bool STAB, int SL>
__global__ __launch_bounds__(256) void scan_chunk_out_kernel(ScanArgs a, ScanChunks c) {
  constexpr int TS = SL + 8, NH = SL / 64, PS = SL + 4, QS = 64 + 8;
  constexpr int Q_BYTES = SL * QS * sizeof(T), P_BYTES = 64 * PS * 4;
  __shared__ __attribute__((aligned(16))) T vt[64 * TS];              // [value][key]
  __shared__ __attribute__((aligned(16))) unsigned char qp_lds[Q_BYTES > P_BYTES ? Q_BYTES : P_BYTES];
  T* qs = reinterpret_cast<T*>(qp_lds);                               // [token][64 of N]
  float* ps = reinterpret_cast<float*>(qp_lds);                       // [token of a half][key] weighted scores
  __shared__ double F_s[SL];
  __shared__ float in_s[SL], m_s[SL], inv_s[64];
  const int v0 = blockIdx.x * 64, h = blockIdx.y, ci = blockIdx.z;
  const int row0 = c.chunks[ci * 4], len = min(c.chunks[ci * 4 + 1], SL);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int nv = min(64, a.V - v0), hk = h / a.per_group;
  const long long ho = static_cast<long long>(ci) * a.H + h;
  const float m0 = STAB ? c.m0[ho] : 0.f;
  load_transposed<T, SL>(static_cast<const T*>(a.v), a.ldv, row0, len, h * a.V + v0, nv, vt);
  if (wid == 0) {
    double F[NH], top[NH];
    float li[NH];
    chunk_gates<NH, STAB>(a, row0, len, h, F, li, top);
#pragma unroll
    for (int i = 0; i < NH; ++i) {
      const int t = lane * NH + i;
      F_s[t] = F[i];
      in_s[t] = li[i];
      m_s[t] = STAB ? static_cast<float>(F[i] + fmax(static_cast<double>(m0), top[i])) : 0.f;
    }
    if constexpr (STAB) {
      const int last = c.chunks[ci * 4 + 3];
      if (blockIdx.x == 0 && lane == 0 && (last & 1))
        a.m[(static_cast<long long>(last >> 1 & 1) * a.slots + c.chunks[ci * 4 + 2]) * a.H + h] =
            static_cast<float>(fmax(c.fl[ho] + m0, c.am[ho]));
    }
  }
  const T* qp = static_cast<const T*>(a.q) + static_cast<long long>(hk) * a.N;
  const T* kp[NH];
#pragma unroll
  for (int k = 0; k < NH; ++k)
    kp[k] = static_cast<const T*>(a.k) + (row0 + min(k * 64 + wid * 16 + fr, len - 1)) * a.ldk + static_cast<long long>(hk) * a.N;
  const float* S0 = c.dS + (ho * a.V + v0 + wid * 16 + fr) * a.N;
  const float* nrm = STAB ? c.dn + ho * a.N : nullptr;
  const bool rows_v = wid * 16 < nv;              // this wave has value rows
  f32x4_t st[NH][NH][4], inter[NH][4];            // [key half][token half][token tile]
  float nq[NH];
#pragma unroll
  for (int k = 0; k < NH; ++k) {
    nq[k] = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      inter[k][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < NH; ++j) st[k][j][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
  }
  for (int n0 = 0; n0 < a.N; n0 += 64) {
    const int nn = min(64, a.N - n0);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2 * NH; ++i) {
      const int idx = tid + i * 256, t = idx >> 3, c8 = (idx & 7) * 8;
      if (c8 < nn) {
        const T* p = qp + (row0 + min(t, len - 1)) * a.ldq + n0 + c8;
        T* d = qs + t * QS + c8;
        *reinterpret_cast<u32x4_t*>(d) = load16(p);
        if constexpr (sizeof(T) == 4) *reinterpret_cast<u32x4_t*>(d + 4) = load16(p + 4);
      }
    }
    __syncthreads();
    for (int n = 0; n < nn; n += 32) {
      Frag<T> kf[NH];
#pragma unroll
      for (int k = 0; k < NH; ++k) kf[k] = load_frag(kp[k] + n0 + n + g * 8);
      float x[8];
      if (rows_v) load8(S0 + n0 + n + g * 8, x);
      else
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = 0.f;
      const WideFrag<T> sf = wide_frag<T>(x);
#pragma unroll
      for (int th = 0; th < NH; ++th)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const Frag<T> qf = load_frag(qs + (th * 64 + j * 16 + fr) * QS + n + g * 8);
#pragma unroll
          for (int k = 0; k < NH; ++k)
            if (k < th || (k == th && j >= wid)) st[k][th][j] = mma(kf[k], qf, st[k][th][j]);
          inter[th][j] = mma(sf, qf, inter[th][j]);
        }
    }
    if constexpr (STAB) {
      const int part = (tid & 3) * 16;
#pragma unroll
      for (int th = 0; th < NH; ++th)
        for (int n = part; n < min(part + 16, nn); ++n) nq[th] += nrm[n0 + n] * to_f32(qs[(th * 64 + (tid >> 2)) * QS + n]);
    }
  }
  Frag<T> vf[SL / 32];
#pragma unroll
  for (int kb = 0; kb < SL / 32; ++kb) vf[kb] = load_frag(vt + (wid * 16 + fr) * TS + kb * 32 + g * 8);
  const float skip = a.skip ? a.skip[h] : 0.f;
#pragma unroll
  for (int th = 0; th < NH; ++th) {
    if (th * 64 >= len) break;                    // block-uniform
    __syncthreads();                              // the query tile, or the scores of the half before, are no longer read
#pragma unroll
    for (int k = 0; k <= th; ++k)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        // weighted scores of keys 64 k + 16 wid + 4 g + r and token 64 th + 16 j + fr
        const int t = th * 64 + j * 16 + fr;
        const double Ft = F_s[t];
        f32x4_t w = st[k][th][j];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int s = k * 64 + wid * 16 + g * 4 + r;
          float e = 0.f;
          if (s <= t && t < len) {
            if constexpr (STAB) e = expf(static_cast<float>(Ft - F_s[s] + static_cast<double>(in_s[s] - m_s[t])));
            else e = expf(static_cast<float>(Ft - F_s[s])) * in_s[s];
          }
          w[r] *= e * a.qscale;
        }
        *reinterpret_cast<f32x4_t*>(ps + (j * 16 + fr) * PS + k * 64 + wid * 16 + g * 4) = w;
      }
    __syncthreads();
    if constexpr (STAB) {
      const int tl = tid >> 2, t = th * 64 + tl;
      float den = 0.f;
#pragma unroll
      for (int k = 0; k <= th; ++k)
#pragma unroll
        for (int i = 0; i < 16; i += 4) {
          const f32x4_t x = *reinterpret_cast<const f32x4_t*>(ps + tl * PS + k * 64 + (tid & 3) * 16 + i);
          den += x[0] + x[1] + x[2] + x[3];
        }
      den += nq[th] * expf(static_cast<float>(F_s[t] + static_cast<double>(m0 - m_s[t]))) * a.qscale;
      den += __shfl_xor(den, 1, 64);
      den += __shfl_xor(den, 2, 64);
      if ((tid & 3) == 0) inv_s[tl] = 1.f / (fmaxf(fabsf(den), expf(-m_s[t])) + 1e-6f);
      __syncthreads();
    }
    if (!rows_v) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int tl = j * 16 + fr, t = th * 64 + tl;
      f32x4_t y = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kb = 0; kb < SL / 32; ++kb)
        if (kb < 2 * th || (kb < 2 * th + 2 && (kb - 2 * th) * 2 <= j)) {
          float x[8];
          load8(ps + tl * PS + kb * 32 + g * 8, x);
          y = mma(vf[kb], wide_frag<T>(x), y);
        }
      if (t >= len) continue;
      y += inter[th][j] * (expf(static_cast<float>(F_s[t] + static_cast<double>(m0 - m_s[t]))) * a.qscale);
      if constexpr (STAB) y *= inv_s[tl];
      const int v = wid * 16 + g * 4;
      if (a.skip) {
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] += skip * to_f32(vt[(v + r) * TS + t]);
      }
      store4(static_cast<T*>(a.out) + (static_cast<long long>(row0 + t) * a.H + h) * a.V + v0 + v, y[0], y[1], y[2], y[3]);
    }
  }
}

template <typename T, bool STAB>
static void launch_scan(const ScanArgs& a, const ScanChunks& c, hipStream_t st) {
  constexpr int SL = sizeof(T) == 2 ? SCAN_CHUNK_BF16 : SCAN_CHUNK_F32;
  const dim3 g1((a.V + 63) / 64, a.H, c.C), block(256);
  const long long quads = static_cast<long long>(a.V) * a.N / 4;
  const dim3 g2(static_cast<unsigned>((quads + 255) / 256) + (STAB ? 1 : 0), a.H, c.nseq);
  hipLaunchKernelGGL((scan_chunk_state_kernel<T, STAB, SL>), g1, block, 0, st, a, c);
  hipLaunchKernelGGL(scan_chunk_pass_kernel<STAB>, g2, block, 0, st, a, c);
  hipLaunchKernelGGL((scan_chunk_out_kernel<T, STAB, SL>), g1, block, 0, st, a, c);
}
void launch_scan_prefill(const ScanArgs& a, const ScanChunks& c, bool f32, hipStream_t st) {
  const bool stab = a.log_in != nullptr;
  if (f32) {
    if (stab) launch_scan<float, true>(a, c, st);
    else launch_scan<float, false>(a, c, st);
  } else {
    if (stab) launch_scan<bf16_t, true>(a, c, st);
    else launch_scan<bf16_t, false>(a, c, st);
  }
}

}  // namespace evgpt
