// Chunk-masked causal attention: a position sees the earlier positions of its own chunk only (chunks of a
// fixed size counted from position 0 of the sequence).  Any head size that is a multiple of 64, any number
// of query heads per key head, either storage type.
//
// Prefill: work items are runs of at most 64 query rows inside ONE chunk, so inside an item the mask is
// plain causal from the chunk's first key; items of all sequences of a pack share one launch.  Four waves,
// sixteen query rows each.  As in attn_prefill.hip the scores are computed transposed (a lane holds keys of
// one query), so the softmax needs two shuffles and the weights are already the operand of the second
// product; here they enter it as two bf16 parts (fp32 attention weights).  Query and key fragments come
// straight from global memory, values through a transposed LDS tile; a block produces 64 value columns.
//
// Decode: the cache of a sequence holds the current chunk in its first pos % cap + 1 slots.
#include "elem.h"
#include "../layered_kernels.h"

namespace evgpt {

constexpr int AC_TS = 64 + 8;

template <typename T>
__global__ __launch_bounds__(256) void attn_chunk_kernel(const T* __restrict__ q, const T* __restrict__ k,
                                                         const T* __restrict__ v, T* __restrict__ o,
                                                         const int* __restrict__ items, int Hq, int Hkv, int D,
                                                         long long kld, float scale, const T* __restrict__ gate, int gate_ld) {
  __shared__ __attribute__((aligned(16))) T vt[64 * AC_TS];
  const int* it = items + blockIdx.x * 4;
  const int q0 = it[0], nq = min(it[1], 64), kv0 = it[2], off = it[3];
  const int h = blockIdx.y, v0 = blockIdx.z * 64, hk = h / (Hq / Hkv);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int t = wid * 16 + fr, tc = min(t, nq - 1);
  const int lim = off + tc;                       // this lane's last visible key
  const int k_end = off + nq;                     // keys the block needs
  const T* qp = q + (static_cast<long long>(q0 + tc) * Hq + h) * D;
  const T* kb = k + static_cast<long long>(kv0) * kld + hk * D;
  const T* vb = v + static_cast<long long>(kv0) * kld + hk * D + v0;
  const int wave_end = min(off + wid * 16 + 16, k_end);   // keys this wave needs
  f32x4_t acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (int k0 = 0; k0 < k_end; k0 += 64) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int idx = tid + i * 256, s = idx & 63, c8 = (idx >> 6) * 8;
      const T* p = vb + min(k0 + s, k_end - 1) * kld + c8;
      T x[8];
      if constexpr (sizeof(T) == 2) *reinterpret_cast<u32x4_t*>(x) = load16(p);
      else {
        *reinterpret_cast<f32x4_t*>(x) = load4(p);
        *reinterpret_cast<f32x4_t*>(x + 4) = load4(p + 4);
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) vt[(c8 + j) * AC_TS + s] = x[j];
    }
    __syncthreads();
    if (k0 >= wave_end) continue;
    f32x4_t st[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) st[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int d = g * 8; d < D; d += 32) {
      const Frag<T> qf = load_frag(qp + d);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        st[i] = mma(load_frag(kb + min(k0 + i * 16 + fr, k_end - 1) * kld + d), qf, st[i]);
    }
    float mt = m;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = k0 + i * 16 + g * 4 + r;
        st[i][r] = key <= lim ? st[i][r] * scale : -INFINITY;
        mt = fmaxf(mt, st[i][r]);
      }
    mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    // key 0 of the chunk is visible to every query, so mt is finite from the first tile on
    const float al = expf(m - mt);
    l *= al;
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] *= al;
    m = mt;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        st[i][r] = expf(st[i][r] - m);
        l += st[i][r];
      }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      float x[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) { x[j] = st[b * 2][j]; x[4 + j] = st[b * 2 + 1][j]; }
      const WideFrag<T> pf = wide_frag<T>(x);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const T* vr = vt + (i * 16 + fr) * AC_TS + b * 32 + g * 4;
        Frag<T> vf;
        if constexpr (sizeof(T) == 2) {
          const u32x2_t lo = *reinterpret_cast<const u32x2_t*>(vr), hi = *reinterpret_cast<const u32x2_t*>(vr + 16);
          vf.v = __builtin_bit_cast(bf16x8_t, u32x4_t{lo[0], lo[1], hi[0], hi[1]});
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) { vf.v[j] = vr[j]; vf.v[4 + j] = vr[16 + j]; }
        }
        acc[i] = mma(vf, pf, acc[i]);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (t >= nq) return;
  float inv = 1.f / l;
  if (gate) inv *= sigmoid_f(to_f32(gate[static_cast<long long>(q0 + t) * gate_ld + h]));
  T* op = o + (static_cast<long long>(q0 + t) * Hq + h) * D + v0;
#pragma unroll
  for (int i = 0; i < 4; ++i)
    store4(op + i * 16 + g * 4, acc[i][0] * inv, acc[i][1] * inv, acc[i][2] * inv, acc[i][3] * inv);
}

void launch_attn_chunk(const void* q, const void* k, const void* v, void* o, const int* items, int n_items, bool f32,
                       int Hq, int Hkv, int D, long long kld, float scale, const void* gate, int gate_ld, hipStream_t st) {
  const dim3 grid(n_items, Hq, D / 64);
  if (f32)
    hipLaunchKernelGGL(attn_chunk_kernel<float>, grid, dim3(256), 0, st, static_cast<const float*>(q),
                       static_cast<const float*>(k), static_cast<const float*>(v), static_cast<float*>(o), items, Hq, Hkv, D,
                       kld, scale, static_cast<const float*>(gate), gate_ld);
  else
    hipLaunchKernelGGL(attn_chunk_kernel<bf16_t>, grid, dim3(256), 0, st, static_cast<const bf16_t*>(q),
                       static_cast<const bf16_t*>(k), static_cast<const bf16_t*>(v), static_cast<bf16_t*>(o), items, Hq, Hkv,
                       D, kld, scale, static_cast<const bf16_t*>(gate), gate_ld);
}

// One query per sequence.  Sixteen lanes per key: lane l holds elements 4 l .. 4 l + 3 of every run of 64, so a
// head of up to 64 E elements is E vectors per lane.
template <typename T, int E>
__global__ __launch_bounds__(256) void attn_chunk_decode_kernel(const T* __restrict__ q, const T* __restrict__ kc,
                                                                const T* __restrict__ vc, T* __restrict__ o,
                                                                const int* __restrict__ row_slot, const int* __restrict__ pos, int Hq, int Hkv, int D,
                                                                int cap, float scale) {
  __shared__ __attribute__((aligned(16))) float so[16][64 * E];
  __shared__ float sm[16], sl[16];
  const int h = blockIdx.x, b = blockIdx.y, hk = h / (Hq / Hkv);
  const int tid = threadIdx.x, l16 = tid & 15, grp = tid >> 4;
  const int len = max(pos[b], 0) % cap + 1;
  const T* qp = q + (static_cast<long long>(b) * Hq + h) * D + l16 * 4;
  const long long base = (static_cast<long long>(row_slot ? row_slot[b] : b) * Hkv + hk) * cap * D + l16 * 4;
  f32x4_t qv[E], ov[E];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    qv[e] = e * 64 < D ? load4(qp + e * 64) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    ov[e] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  float m = -INFINITY, l = 0.f;
  for (int key = grp; key < len; key += 16) {
    const T* kp = kc + base + static_cast<long long>(key) * D;
    const T* vp = vc + base + static_cast<long long>(key) * D;
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < E; ++e)
      if (e * 64 < D) {
        const f32x4_t kk = load4(kp + e * 64);
#pragma unroll
        for (int i = 0; i < 4; ++i) s += kk[i] * qv[e][i];
      }
    s = group_sum<16>(s) * scale;
    const float mn = fmaxf(m, s), al = expf(m - mn), p = expf(s - mn);
    l = l * al + p;
#pragma unroll
    for (int e = 0; e < E; ++e)
      if (e * 64 < D) ov[e] = ov[e] * al + load4(vp + e * 64) * p;
    m = mn;
  }
#pragma unroll
  for (int e = 0; e < E; ++e) *reinterpret_cast<f32x4_t*>(&so[grp][e * 64 + l16 * 4]) = ov[e];
  if (l16 == 0) { sm[grp] = m; sl[grp] = l; }
  __syncthreads();
  float mm = -INFINITY, ll = 0.f;
  for (int i = 0; i < 16; ++i) mm = fmaxf(mm, sm[i]);
  float c[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    c[i] = sm[i] == -INFINITY ? 0.f : expf(sm[i] - mm);
    ll += sl[i] * c[i];
  }
  for (int d = tid; d < D; d += 256) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) s += so[i][d] * c[i];
    o[(static_cast<long long>(b) * Hq + h) * D + d] = from_f32<T>(s / ll);
  }
}

template <typename T>
static void launch_decode(const void* q, const void* kc, const void* vc, void* o, const int* row_slot, const int* pos, int B, int Hq,
                          int Hkv, int D, int cap, float scale, hipStream_t st) {
  const dim3 grid(Hq, B), block(256);
  const T *qt = static_cast<const T*>(q), *kt = static_cast<const T*>(kc), *vt = static_cast<const T*>(vc);
  T* ot = static_cast<T*>(o);
  if (D <= 64) hipLaunchKernelGGL((attn_chunk_decode_kernel<T, 1>), grid, block, 0, st, qt, kt, vt, ot, row_slot, pos, Hq, Hkv, D, cap, scale);
  else if (D <= 128) hipLaunchKernelGGL((attn_chunk_decode_kernel<T, 2>), grid, block, 0, st, qt, kt, vt, ot, row_slot, pos, Hq, Hkv, D, cap, scale);
  else if (D <= 256) hipLaunchKernelGGL((attn_chunk_decode_kernel<T, 4>), grid, block, 0, st, qt, kt, vt, ot, row_slot, pos, Hq, Hkv, D, cap, scale);
  else hipLaunchKernelGGL((attn_chunk_decode_kernel<T, 8>), grid, block, 0, st, qt, kt, vt, ot, row_slot, pos, Hq, Hkv, D, cap, scale);
}
void launch_attn_chunk_decode(const void* q, const void* k_cache, const void* v_cache, void* o, const int* row_slot, const int* pos,
                              bool f32, int B, int Hq, int Hkv, int D, int cap, float scale, hipStream_t st) {
  if (f32) launch_decode<float>(q, k_cache, v_cache, o, row_slot, pos, B, Hq, Hkv, D, cap, scale, st);
  else launch_decode<bf16_t>(q, k_cache, v_cache, o, row_slot, pos, B, Hq, Hkv, D, cap, scale, st);
}

}  // namespace evgpt
