// Latent attention: keys and values of every head are linear in one short row per token, which is all the cache
// holds ([slots][cap][R], zero-padded columns).
//
//   prep     a projection's rows -> normed query latents, normed key / value latents straight into the cache;
//   gather   cached rows of several sequences into one buffer, which a long prompt expands to keys and values;
//   heads    a small product per head, y[row][h] = W[h] x[row][h]: it takes a query into the latent space (so that
//            scores are products with cached rows) and an attended latent out of it;
//   attend   attention of single queries over the cached rows: all heads share them, so the scores of sixteen
//            heads are one MFMA tile and every row is read once per sixteen heads.
//
// attend: a block takes sixteen heads of one query and a run of keys; its four waves take 32 keys at a time, each with
// its own softmax state, so that the loop has no barrier.  A wave's keys are MFMA operands straight from global memory
// for the scores; the same registers go to LDS, from where the transposing read gives the operand of the second
// product.  Scores are computed transposed (a lane holds keys of one head), as in attn_prefill.hip, so the weights
// are already the other operand; they enter as two bf16 parts.
#include "src_rows.h"

namespace evgpt {

// ---------------------------------------------------------------- prep
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrepArgs a, int rows) {
  const int lane = threadIdx.x & 63;
  const long long row = blockIdx.x * 4ll + (threadIdx.x >> 6);
  if (row >= rows) return;
  if (a.q_out) latent_row(a.src, row, a.q_col, a.nq, a.Q, a.qw, a.eps, static_cast<T*>(a.q_out) + row * a.Q, lane);
  if (a.cache && !(a.live && !a.live[row])) {
    const long long slot = a.row_slot ? a.row_slot[row] : row;
    const int p = min(max(a.row_pos[row], 0), a.cap - 1);
    latent_row(a.src, row, a.c_col, a.nc, a.R, a.cw, a.eps, static_cast<T*>(a.cache) + (slot * a.cap + p) * a.R, lane);
  }
}
void launch_latent_prep(const LatentPrepArgs& a, bool f32, int rows, hipStream_t st) {
  const dim3 grid((rows + 3) / 4), block(256);
  if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, grid, block, 0, st, a, rows);
  else hipLaunchKernelGGL(latent_prep_kernel<bf16_t>, grid, block, 0, st, a, rows);
}

// copies [n][4] of {slot, first position, first buffer row, count}; rows are vec 16-byte chunks
__global__ __launch_bounds__(256) void latent_gather_kernel(const u32x4_t* __restrict__ cache, u32x4_t* __restrict__ buf,
                                                            const int* __restrict__ copies, int cap, int vec) {
  const int* c = copies + blockIdx.y * 4;
  const u32x4_t* s = cache + (static_cast<long long>(c[0]) * cap + c[1]) * vec;
  u32x4_t* d = buf + static_cast<long long>(c[2]) * vec;
  const long long n = static_cast<long long>(c[3]) * vec;
  for (long long i = blockIdx.x * 256ll + threadIdx.x; i < n; i += gridDim.x * 256ll) d[i] = s[i];
}
void launch_latent_gather(const void* cache, void* buf, const int* copies, int n, bool f32, int cap, int R, hipStream_t st) {
  hipLaunchKernelGGL(latent_gather_kernel, dim3(256, n), dim3(256), 0, st, static_cast<const u32x4_t*>(cache),
                     static_cast<u32x4_t*>(buf), copies, cap, R * (f32 ? 4 : 2) / 16);
}

// ---------------------------------------------------------------- key splits of attend
// Keys per split: at least LT_MIN, whole multiples of it, so that short contexts use few splits.
constexpr int LT_MIN = 128;
__device__ __forceinline__ int split_keys(int len, int nsplit) {
  const int per = (len + nsplit - 1) / nsplit;
  return (per + LT_MIN - 1) / LT_MIN * LT_MIN;
}
__device__ __forceinline__ int latent_len(const int* pos, int row, int cap) { return min(max(pos[row] + 1, 1), cap); }

// ---------------------------------------------------------------- heads
// Block: sixteen rows, one head, 64 outputs (a wave has sixteen of them) or -- NARROW -- sixteen outputs with the
// contraction shared by the waves.  The rows' inputs are staged in LDS: columns of SrcRows, or the merge of attend's splits.
template <typename T, bool MERGE, bool NARROW>
__global__ __launch_bounds__(256) void head_linear_kernel(HeadLinearArgs a, int rows) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ __attribute__((aligned(16))) float part[NARROW ? 3 : 1][64][4];
  T* xs = reinterpret_cast<T*>(smem);
  const int K = a.K, ldx = K + 16 / static_cast<int>(sizeof(T));
  const int h = blockIdx.y, r0 = blockIdx.z * 16, nr = min(rows - r0, 16);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int n0 = NARROW ? blockIdx.x * 16 : blockIdx.x * 64 + wid * 16;
  const T* wp = static_cast<const T*>(a.w) + (static_cast<long long>(h) * a.N + min(n0 + fr, a.N - 1)) * K + g * 8;
  for (int r = wid; r < 16; r += 4) {
    if (r >= nr) {
      const float z[8] = {0, 0, 0, 0, 0, 0, 0, 0};
      for (int c = lane * 8; c < K; c += 512) store8(xs + r * ldx + c, z);
      continue;
    }
    const int row = r0 + r;
    if constexpr (MERGE) {
      const int len = latent_len(a.pos, row, a.cap), per = split_keys(len, a.nsplit), used = (len + per - 1) / per;
      const float* ml = a.part_ml + (static_cast<long long>(row) * a.H + h) * a.nsplit * 2;
      const float* po = a.part_o + (static_cast<long long>(row) * a.H + h) * a.nsplit * K;
      float mx = -INFINITY;
      for (int s = lane; s < used; s += 64) mx = fmaxf(mx, ml[2 * s]);
      mx = wave_max(mx);
      float l = 0.f;
      for (int s = lane; s < used; s += 64) l += __builtin_amdgcn_exp2f(ml[2 * s] - mx) * ml[2 * s + 1];
      const float inv = 1.f / wave_sum(l);
      for (int c = lane * 8; c < K; c += 512) {
        float o[8] = {0, 0, 0, 0, 0, 0, 0, 0};
        for (int s0 = 0; s0 < used; s0 += 4) {
          float v[4][8], f[4];
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            const int s = min(s0 + u, used - 1);
            load8(po + static_cast<long long>(s) * K + c, v[u]);
            f[u] = s0 + u < used ? __builtin_amdgcn_exp2f(ml[2 * s] - mx) : 0.f;
          }
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 8; ++i) o[i] += f[u] * v[u][i];
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] *= inv;
        store8(xs + r * ldx + c, o);
      }
    } else {
      for (int c = lane * 8; c < K; c += 512) {
        float v[8];
        src8(a.x, row, a.x_col + h * K + c, v);
        store8(xs + r * ldx + c, v);
      }
    }
  }
  __syncthreads();
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  const T* xp = xs + fr * ldx + g * 8;
#pragma unroll 4
  for (int k = NARROW ? wid * 32 : 0; k < K; k += NARROW ? 128 : 32) acc = mma(load_frag(wp + k), load_frag(xp + k), acc);
  if constexpr (NARROW) {
    if (wid > 0) *reinterpret_cast<f32x4_t*>(part[wid - 1][lane]) = acc;
    __syncthreads();
    if (wid > 0) return;
#pragma unroll
    for (int w = 0; w < 3; ++w) acc += *reinterpret_cast<const f32x4_t*>(part[w][lane]);
  }
  const int n = n0 + g * 4;                       // N % 16 == 0: all four or none
  if (fr >= nr || n >= a.N) return;
  const long long row = r0 + fr;
  if (a.gate.p) acc *= sigmoid_f(src1(a.gate, row, a.gcol + h));
  store4(static_cast<T*>(a.y) + (row * a.H + h) * a.N + n, acc[0], acc[1], acc[2], acc[3]);
}
template <typename T, bool MERGE>
static void launch_heads(const HeadLinearArgs& a, int rows, hipStream_t st) {
  const int tiles = (rows + 15) / 16;
  const size_t lds = 16ull * (a.K * sizeof(T) + 16);
  // enough blocks for the chip from the 64-wide tiles, or the narrow ones
  const int wide = (a.N + 63) / 64;
  if (static_cast<long long>(wide) * a.H * tiles >= 192)
    hipLaunchKernelGGL((head_linear_kernel<T, MERGE, false>), dim3(wide, a.H, tiles), dim3(256), lds, st, a, rows);
  else
    hipLaunchKernelGGL((head_linear_kernel<T, MERGE, true>), dim3(a.N / 16, a.H, tiles), dim3(256), lds, st, a, rows);
}
void launch_head_linear(const HeadLinearArgs& a, bool f32, int rows, hipStream_t st) {
  if (a.part_o) launch_heads<bf16_t, true>(a, rows, st);
  else if (f32) launch_heads<float, false>(a, rows, st);
  else launch_heads<bf16_t, false>(a, rows, st);
}

// ---------------------------------------------------------------- attend
// byte offset of 16-byte chunk `ch` of key `row` in a wave's [32][R] image: the swizzles of attn_common.h
template <int R>
__device__ __forceinline__ int lt_off(int row, int ch) {
  const int x = R == 64 ? ((row >> 1) & 3) << 1 : (row & 7) << 1;
  return row * (R * 2) + ((ch ^ x) << 4);
}

template <int R>
__global__ __launch_bounds__(256, 1) void latent_attend_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ cache,
                                                               float* __restrict__ part_o, float* __restrict__ part_ml,
                                                               const int* __restrict__ row_slot, const int* __restrict__ pos,
                                                               int H, int cap, float scale_log2e) {
  constexpr int KS = R / 32, RT = R / 16;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];      // [4 waves][32 keys][R] bf16, or [16 heads][R] fp32
  __shared__ float s_m[4][16], s_l[4][16];
  const int split = blockIdx.x, nsplit = gridDim.x, h0 = blockIdx.y * 16, b = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int len = latent_len(pos, b, cap), per = split_keys(len, nsplit);
  const int k_begin = split * per, k_end = min(len, k_begin + per);
  if (k_begin >= len) return;
  const bf16_t* cb = cache + static_cast<long long>(row_slot ? row_slot[b] : b) * cap * R;
  unsigned char* img = smem + wid * (32 * R * 2);
  const bf16_t* qp = q + (static_cast<long long>(b) * H + min(h0 + fr, H - 1)) * R + g * 8;
  bf16x8_t qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) qf[ks] = __builtin_bit_cast(bf16x8_t, load16(qp + ks * 32));
  f32x4_t o[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) o[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  u32x4_t kr[2][KS];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const bf16_t* p = cb + static_cast<long long>(min(k0 + n * 16 + fr, len - 1)) * R + g * 8;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) kr[n][ks] = load16(p + ks * 32);
    }
  };
  int k0 = k_begin + wid * 32;
  if (k0 < k_end) fetch(k0);
  for (; k0 < k_end; k0 += 128) {
    f32x4_t st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        *reinterpret_cast<u32x4_t*>(img + lt_off<R>(n * 16 + fr, ks * 4 + g)) = kr[n][ks];
        st[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kr[n][ks]), qf[ks], st[n], 0, 0, 0);
      }
    if (k0 + 128 < k_end) fetch(k0 + 128);
    float mt = m;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (k0 + n * 16 + g * 4 + r >= k_end) st[n][r] = -INFINITY;
        mt = fmaxf(mt, st[n][r]);
      }
    mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));      // finite: key k0 is there
    if (__builtin_amdgcn_ballot_w64(mt != m) != 0) {
      const float al = __builtin_amdgcn_exp2f((m - mt) * scale_log2e);
      l *= al;
#pragma unroll
      for (int i = 0; i < RT; ++i) o[i] *= al;
      m = mt;
    }
    const float ms = m * scale_log2e;
    u32x4_t hi, lo;
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      float e[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) { e[r] = __builtin_amdgcn_exp2f(fmaf(st[n][r], scale_log2e, -ms)); l += e[r]; }
      hi[n * 2] = pack_bf16x2(e[0], e[1]);
      hi[n * 2 + 1] = pack_bf16x2(e[2], e[3]);
      lo[n * 2] = pack_bf16x2(e[0] - bf16lo(hi[n * 2]), e[1] - bf16hi(hi[n * 2]));
      lo[n * 2 + 1] = pack_bf16x2(e[2] - bf16lo(hi[n * 2 + 1]), e[3] - bf16hi(hi[n * 2 + 1]));
    }
    const bf16x8_t ph = __builtin_bit_cast(bf16x8_t, hi), pl = __builtin_bit_cast(bf16x8_t, lo);
    // a wave's LDS operations execute in order; the compiler has to keep them in this order too
    asm volatile("" ::: "memory");
    const int q4 = fr >> 2, p4 = fr & 3, r0 = g * 4 + q4;
#pragma unroll
    for (int t = 0; t < RT; ++t) {
      const int ch = t * 2 + (p4 >> 1);
      const s16x4_t va = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
          (s16x4_t __attribute__((address_space(3)))*)(img + lt_off<R>(r0, ch) + 8 * (p4 & 1)));
      const s16x4_t vb = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
          (s16x4_t __attribute__((address_space(3)))*)(img + lt_off<R>(r0 + 16, ch) + 8 * (p4 & 1)));
      typedef __attribute__((ext_vector_type(8))) short s16x8_t;
      const s16x8_t vv = {va[0], va[1], va[2], va[3], vb[0], vb[1], vb[2], vb[3]};
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vv), pl, o[t], 0, 0, 0);
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vv), ph, o[t], 0, 0, 0);
    }
    asm volatile("" ::: "memory");
  }
  // merge of the four waves: a wave without keys has m = -inf and weight 0
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  float* so = reinterpret_cast<float*>(img);
#pragma unroll
  for (int t = 0; t < RT; ++t) *reinterpret_cast<f32x4_t*>(so + fr * R + ((t * 16 + g * 4) ^ ((fr & 7) << 2))) = o[t];
  if (g == 0) { s_m[wid][fr] = m; s_l[wid][fr] = l; }
  __syncthreads();
  for (int i = tid * 4; i < 16 * R; i += 1024) {
    const int hh = i / R, c = i % R;
    if (h0 + hh >= H) break;
    float mx = s_m[0][hh];
#pragma unroll
    for (int w = 1; w < 4; ++w) mx = fmaxf(mx, s_m[w][hh]);
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
    float ll = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f((s_m[w][hh] - mx) * scale_log2e);
      ll += f * s_l[w][hh];
      s += *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const float*>(smem + w * (32 * R * 2)) + hh * R + (c ^ ((hh & 7) << 2))) * f;
    }
    const long long slot = (static_cast<long long>(b) * H + h0 + hh) * nsplit + split;
    *reinterpret_cast<f32x4_t*>(part_o + slot * R + c) = s;
    if (c == 0) { part_ml[slot * 2] = mx * scale_log2e; part_ml[slot * 2 + 1] = ll; }
  }
}
template <int R>
static void launch_attend(const bf16_t* q, const bf16_t* cache, float* part_o, float* part_ml, const int* row_slot,
                          const int* pos, int rows, int H, int cap, int nsplit, float scale, hipStream_t st) {
  constexpr int lds = 4 * 32 * R * 2;
  static const bool attr = [] {
    return hipFuncSetAttribute(reinterpret_cast<const void*>(latent_attend_kernel<R>),
                               hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
  }();
  (void)attr;
  hipLaunchKernelGGL(latent_attend_kernel<R>, dim3(nsplit, (H + 15) / 16, rows), dim3(256), lds, st, q, cache, part_o, part_ml,
                     row_slot, pos, H, cap, scale * 1.4426950408889634f);
}
void launch_latent_attend(const bf16_t* q, const bf16_t* cache, float* part_o, float* part_ml, const int* row_slot,
                          const int* pos, int rows, int H, int R, int cap, int nsplit, float scale, hipStream_t st) {
#define EVGPT_ATTEND(R_) launch_attend<R_>(q, cache, part_o, part_ml, row_slot, pos, rows, H, cap, nsplit, scale, st)
  if (R == 64) EVGPT_ATTEND(64);
  else if (R == 128) EVGPT_ATTEND(128);
  else if (R == 256) EVGPT_ATTEND(256);
  else if (R == 384) EVGPT_ATTEND(384);
  else EVGPT_ATTEND(512);
#undef EVGPT_ATTEND
}

}  // namespace evgpt
