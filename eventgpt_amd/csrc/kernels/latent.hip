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
// attend: a block takes 16 or 32 heads of one query and a run of keys.  Tiles of 64 keys come straight into LDS, two
// buffers; for every sixteen heads there are four waves.  A wave scores sixteen of the tile's keys (transposed: a
// lane holds keys of one head, as in attn_prefill.hip), the four agree on the maximum, and their weights go through LDS as
// two bf16 parts each -- a lane's four are half of the other operand as they are --, after which the wave multiplies all 64
// weights with its quarter of the columns, read from the tile with the transposing read.  No wave holds more than a
// quarter of a head's output, and nothing is left to merge but the splits.
#include "src_rows.h"

namespace evgpt {

// ---------------------------------------------------------------- prep
// A block per row.  The first chunk of either section stays in registers, further ones are read again.
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrepArgs a) {
  __shared__ float red[8];
  const long long row = blockIdx.x;
  const int tid = threadIdx.x, Q = a.q_out ? a.Q : 0, R = a.cache && !(a.live && !a.live[row]) ? a.R : 0;
  float vq[8], vc[8], sq = 0.f, sc = 0.f;
  // the latents' chunks go to the last threads first: they are free where the query section is short of a full pass
  const int tc = 255 - tid;
  for (int c = tid * 8; c < Q; c += 2048) {
    float v[8];
    section8(a.src, row, a.q_col, a.nq, c, v);
    sq += sumsq8(v);
    if (c == tid * 8)
#pragma unroll
      for (int i = 0; i < 8; ++i) vq[i] = v[i];
  }
  for (int c = tc * 8; c < R; c += 2048) {
    float v[8];
    section8(a.src, row, a.c_col, a.nc, c, v);
    sc += sumsq8(v);
    if (c == tc * 8)
#pragma unroll
      for (int i = 0; i < 8; ++i) vc[i] = v[i];
  }
  sq = wave_sum(sq);
  sc = wave_sum(sc);
  if ((tid & 63) == 0) { red[tid >> 6] = sq; red[4 + (tid >> 6)] = sc; }
  __syncthreads();
  const float rq = rsqrtf((red[0] + red[1] + red[2] + red[3]) / static_cast<float>(a.nq) + a.eps);
  const float rc = rsqrtf((red[4] + red[5] + red[6] + red[7]) / static_cast<float>(a.nc) + a.eps);
  auto put = [&](int c, int first, const float (&kept)[8], int col, int n, const float* w, float r, T* out) {
    float v[8], g[8];
    if (c == first) {
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = kept[i];
    } else {
      section8(a.src, row, col, n, c, v);
    }
    load8(w + c, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= r * g[i];
    store8(out + c, v);
  };
  for (int c = tid * 8; c < Q; c += 2048) put(c, tid * 8, vq, a.q_col, a.nq, a.qw, rq, static_cast<T*>(a.q_out) + row * a.Q);
  if (R == 0) return;
  const long long slot = a.row_slot ? a.row_slot[row] : row;
  const int p = min(max(a.row_pos[row], 0), a.cap - 1);
  T* out = static_cast<T*>(a.cache) + (slot * a.cap + p) * a.R;
  for (int c = tc * 8; c < R; c += 2048) put(c, tc * 8, vc, a.c_col, a.nc, a.cw, rc, out);
}
void launch_latent_prep(const LatentPrepArgs& a, bool f32, int rows, hipStream_t st) {
  if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(rows), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_prep_kernel<bf16_t>, dim3(rows), dim3(256), 0, st, a);
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
// Keys per split: whole tiles of LT_KEYS, so that short contexts use few splits.
constexpr int LT_KEYS = 64;
__device__ __forceinline__ int split_keys(int len, int nsplit) {
  const int per = (len + nsplit - 1) / nsplit;
  return (per + LT_KEYS - 1) / LT_KEYS * LT_KEYS;
}
__device__ __forceinline__ int latent_len(const int* pos, int row, int cap) { return min(max(pos[row] + 1, 1), cap); }

// ---------------------------------------------------------------- heads
// Block: sixteen rows and one head.  WIDE: 64 outputs, 16 of them per wave column; otherwise 16.  The contraction is shared
// by KW waves per column.  The rows' inputs are staged in LDS: columns of SrcRows, or the merge of attend's splits (a wave
// per row).
template <typename T, bool MERGE, bool WIDE, int KW>
__global__ __launch_bounds__((WIDE ? 256 : 64) * KW) void head_linear_kernel(HeadLinearArgs a, int rows) {
  constexpr int WN = WIDE ? 4 : 1, NT = 64 * WN * KW;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ __attribute__((aligned(16))) float part[KW > 1 ? KW - 1 : 1][WN][64][4];
  T* xs = reinterpret_cast<T*>(smem);
  const int K = a.K, ldx = K + 16 / static_cast<int>(sizeof(T));
  const int h = blockIdx.y, r0 = blockIdx.z * 16, nr = min(rows - r0, 16);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, fr = lane & 15, g = lane >> 4;
  const int wn = wid % WN, wk = wid / WN;
  const int n0 = blockIdx.x * (16 * WN) + wn * 16;
  const T* wp = static_cast<const T*>(a.w) + (static_cast<long long>(h) * a.N + min(n0 + fr, a.N - 1)) * K + g * 8;
  if constexpr (MERGE) {
    // A wave takes a whole row (WIDE), or its share of the columns of every row with four groups of lanes on different
    // splits.  Maxima and sums (a lane per split, at most 64) are on their way together with the first partial rows.
    constexpr int LG = WIDE ? 1 : 4, CL = 64 / LG, U = WIDE ? 8 : 4, STEP = WIDE ? 512 : CL * 8 * KW;
    const int sg = lane / CL, c_lane = ((WIDE ? 0 : wk * CL) + lane % CL) * 8;
    for (int r = WIDE ? wid : 0; r < 16; r += WIDE ? NT / 64 : 1) {
      if (r >= nr) {
        const float z[8] = {0, 0, 0, 0, 0, 0, 0, 0};
        for (int c = c_lane; c < K; c += STEP)
          if (sg == 0) store8(xs + r * ldx + c, z);
        continue;
      }
      const int row = r0 + r;
      const int len = latent_len(a.pos, row, a.cap), per = split_keys(len, a.nsplit), used = (len + per - 1) / per;
      const float* ml = a.part_ml + (static_cast<long long>(row) * a.H + h) * a.nsplit * 2;
      const float* po = a.part_o + (static_cast<long long>(row) * a.H + h) * a.nsplit * K;
      float m = ml[2 * min(lane, used - 1)], f = 0.f, inv = 0.f;
      const float l = ml[2 * min(lane, used - 1) + 1];
      for (int c0 = 0; c0 < K; c0 += STEP) {
        const int c = min(c0 + c_lane, K - 8);
        float o[8] = {0, 0, 0, 0, 0, 0, 0, 0};
        for (int s0 = 0; s0 < used; s0 += LG * U) {
          float v[U][8];
#pragma unroll
          for (int u = 0; u < U; ++u) load8(po + static_cast<long long>(min(s0 + u * LG + sg, used - 1)) * K + c, v[u]);
          if (c0 == 0 && s0 == 0) {
            if (lane >= used) m = -INFINITY;
            f = __builtin_amdgcn_exp2f(m - wave_max(m));   // 0 past the last split
            inv = 1.f / wave_sum(lane < used ? f * l : 0.f);
          }
#pragma unroll
          for (int u = 0; u < U; ++u) {
            const int s = s0 + u * LG + sg;
            const float t = __shfl(f, s & 63, 64), fu = s < used ? t : 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) o[i] += fu * v[u][i];
          }
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if constexpr (LG == 4) {
            o[i] += __shfl_xor(o[i], 16, 64);
            o[i] += __shfl_xor(o[i], 32, 64);
          }
          o[i] *= inv;
        }
        if (sg == 0 && c0 + c_lane < K) store8(xs + r * ldx + c, o);
      }
    }
  } else {
    const int per = K >> 3;
    for (int i = tid; i < 16 * per; i += NT) {
      const int r = i / per, c = i % per * 8;
      float v[8] = {0, 0, 0, 0, 0, 0, 0, 0};
      if (r < nr) src8(a.x, r0 + r, a.x_col + h * K + c, v);
      store8(xs + r * ldx + c, v);
    }
  }
  __syncthreads();
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  const T* xp = xs + fr * ldx + g * 8;
#pragma unroll 4
  for (int k = wk * 32; k < K; k += KW * 32) acc = mma(load_frag(wp + k), load_frag(xp + k), acc);
  if constexpr (KW > 1) {
    if (wk > 0) *reinterpret_cast<f32x4_t*>(part[wk - 1][wn][lane]) = acc;
    __syncthreads();
    if (wk > 0) return;
#pragma unroll
    for (int w = 0; w < KW - 1; ++w) acc += *reinterpret_cast<const f32x4_t*>(part[w][wn][lane]);
  }
  const int n = n0 + g * 4;                       // N % 16 == 0: all four or none
  if (fr >= nr || n >= a.N) return;
  const long long row = r0 + fr;
  if (a.gate.p) acc *= sigmoid_f(src1(a.gate, row, a.gcol + h));
  store4(static_cast<T*>(a.y) + (row * a.H + h) * a.N + n, acc[0], acc[1], acc[2], acc[3]);
}
template <typename T, bool MERGE>
static void launch_heads(const HeadLinearArgs& a, int rows, hipStream_t st) {
  const int tiles = (rows + 15) / 16, wide = (a.N + 63) / 64;
  const size_t lds = 16ull * (a.K * sizeof(T) + 16);
  // the 64-wide tiles where they are enough blocks, or where inputs are merged (the narrow ones merge four times as often)
  if (MERGE && rows > 2)
    hipLaunchKernelGGL((head_linear_kernel<T, MERGE, true, 4>), dim3(wide, a.H, tiles), dim3(1024), lds, st, a, rows);
  else if (static_cast<long long>(wide) * a.H * tiles >= 192)
    hipLaunchKernelGGL((head_linear_kernel<T, MERGE, true, 1>), dim3(wide, a.H, tiles), dim3(256), lds, st, a, rows);
  else
    hipLaunchKernelGGL((head_linear_kernel<T, MERGE, false, 4>), dim3(a.N / 16, a.H, tiles), dim3(256), lds, st, a, rows);
}
void launch_head_linear(const HeadLinearArgs& a, bool f32, int rows, hipStream_t st) {
  if (a.part_o) launch_heads<bf16_t, true>(a, rows, st);
  else if (f32) launch_heads<float, false>(a, rows, st);
  else launch_heads<bf16_t, false>(a, rows, st);
}

// ---------------------------------------------------------------- attend
// A tile [64][R]: 16-byte chunk ch of a key's row lies at ch ^ x, the swizzles of attn_common.h.  x is below 16 (R = 64:
// below 8), so chunks 16 apart (8 apart) keep their distance and one address serves all of them.
// a barrier that leaves the next tile's loads in flight (__syncthreads would wait for them)
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

template <int R> __device__ __forceinline__ int lt_swizzle(int row) { return R == 64 ? ((row >> 1) & 3) << 1 : (row & 7) << 1; }

__device__ __forceinline__ void latent_to_lds16(const unsigned char* src, int bytes, unsigned char* lds, int voff) {
  const auto rs = __builtin_amdgcn_make_buffer_rsrc(const_cast<unsigned char*>(src), 0, bytes, 0x00020000);
  __builtin_amdgcn_raw_ptr_buffer_load_lds(rs, (void __attribute__((address_space(3)))*)lds, 16, voff, 0, 0, 0);
}

// HT: head tiles of sixteen per block (four waves each)
template <int R, int HT>
__global__ __launch_bounds__(256 * HT) void latent_attend_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ cache,
                                                                 float* __restrict__ part_o, float* __restrict__ part_ml,
                                                                 const int* __restrict__ row_slot, const int* __restrict__ pos,
                                                                 int H, int cap, float scale_log2e) {
  constexpr int KS = R / 32, CT = R / 64;              // contraction steps of the scores; column tiles of a wave
  constexpr int TILE = LT_KEYS * R * 2, NI = TILE / 1024 / (4 * HT);     // staging instructions per wave and tile
  constexpr int CPR = R / 8;
  static_assert(NI >= 1, "a tile is at least one staging instruction per wave");
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // [2 tiles], weights [HT][4][64 lanes] of 16 bytes
  __shared__ float s_max[HT][4][16], s_sum[HT][4][16];
  const int split = blockIdx.x, nsplit = gridDim.x, b = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, fr = lane & 15, g = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6), ht = wid >> 2, w4 = wid & 3;
  const int h0 = (blockIdx.z * HT + ht) * 16;
  const int len = latent_len(pos, b, cap), per = split_keys(len, nsplit);
  const int k_begin = split * per, k_end = min(len, k_begin + per);
  if (k_begin >= len) return;
  const unsigned char* cb = reinterpret_cast<const unsigned char*>(cache + static_cast<long long>(row_slot ? row_slot[b] : b) * cap * R);
  unsigned char* weights = smem + 2 * TILE + ht * 4096;
  int voff[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int idx = (wid * NI + i) * 64 + lane, row = idx / CPR;
    voff[i] = row * (R * 2) + (((idx % CPR) ^ lt_swizzle<R>(row)) << 4);
  }
  // (keys past the end lie past the descriptor's range and arrive as zeros)
  auto stage = [&](int buf, int k0) {
    unsigned char* d = smem + buf * TILE + wid * NI * 1024;
#pragma unroll
    for (int i = 0; i < NI; ++i) latent_to_lds16(cb + static_cast<long long>(k0) * (R * 2), (k_end - k0) * (R * 2), d + i * 1024, voff[i]);
  };
  stage(0, k_begin);
  const bf16_t* qp = q + (static_cast<long long>(b) * H + min(h0 + fr, H - 1)) * R + g * 8;
  bf16x8_t qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) qf[ks] = __builtin_bit_cast(bf16x8_t, load16(qp + ks * 32));
  f32x4_t o[CT];
#pragma unroll
  for (int i = 0; i < CT; ++i) o[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  constexpr int CG = R == 64 ? 8 : 16;            // chunks a swizzle stays within
  constexpr int KA = CG / 4;                      // addresses of the score operand (steps of four chunks)
  int kaddr[KA];
#pragma unroll
  for (int i = 0; i < KA; ++i) kaddr[i] = (w4 * 16 + fr) * (R * 2) + (((i * 4 + g) ^ lt_swizzle<R>(w4 * 16 + fr)) << 4);
  const int q4 = fr >> 2, p4 = fr & 3, vrow = g * 4 + q4;      // (rows 16 and 32 further have the same swizzle)
  int vaddr[CT];
#pragma unroll
  for (int t = 0; t < CT; ++t)
    vaddr[t] = vrow * (R * 2) + ((((w4 * CT + t) * 2 + (p4 >> 1)) ^ lt_swizzle<R>(vrow)) << 4) + 8 * (p4 & 1);
  int buf = 0;
  for (int k0 = k_begin; k0 < k_end; k0 += LT_KEYS, buf ^= 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                              // the tile has landed; the other buffer and the weights are free
    if (k0 + LT_KEYS < k_end) stage(buf ^ 1, k0 + LT_KEYS);
    const unsigned char* tile = smem + buf * TILE;
    f32x4_t s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ks += 2) {
      const bf16x8_t ka = *reinterpret_cast<const bf16x8_t*>(tile + kaddr[ks % KA] + ks / KA * (CG * 16));
      const bf16x8_t kb = *reinterpret_cast<const bf16x8_t*>(tile + kaddr[(ks + 1) % KA] + (ks + 1) / KA * (CG * 16));
      s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, qf[ks], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kb, qf[ks + 1], s1, 0, 0, 0);
    }
    s0 += s1;
    float mt = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (k0 + w4 * 16 + g * 4 + r >= k_end) s0[r] = -INFINITY;
      mt = fmaxf(mt, s0[r]);
    }
    mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    if (g == 0) s_max[ht][w4][fr] = mt;
    lds_barrier();
    mt = m;                                       // the tile's first key is there: finite
#pragma unroll
    for (int w = 0; w < 4; ++w) mt = fmaxf(mt, s_max[ht][w][fr]);
    const bool moved = __builtin_amdgcn_ballot_w64(mt != m) != 0;
    const float al = __builtin_amdgcn_exp2f((m - mt) * scale_log2e);
    m = mt;
    const float ms = m * scale_log2e;
    float e[4], sum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) { e[r] = __builtin_amdgcn_exp2f(fmaf(s0[r], scale_log2e, -ms)); sum += e[r]; }
    l = l * al + sum;
    u32x4_t p;
    p[0] = pack_bf16x2(e[0], e[1]);
    p[1] = pack_bf16x2(e[2], e[3]);
    p[2] = pack_bf16x2(e[0] - bf16lo(p[0]), e[1] - bf16hi(p[0]));
    p[3] = pack_bf16x2(e[2] - bf16lo(p[1]), e[3] - bf16hi(p[1]));
    *reinterpret_cast<u32x4_t*>(weights + w4 * 1024 + lane * 16) = p;
    if (moved)
#pragma unroll
      for (int i = 0; i < CT; ++i) o[i] *= al;
    lds_barrier();
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const u32x4_t pa = *reinterpret_cast<const u32x4_t*>(weights + (2 * s) * 1024 + lane * 16);
      const u32x4_t pb = *reinterpret_cast<const u32x4_t*>(weights + (2 * s + 1) * 1024 + lane * 16);
      const bf16x8_t ph = __builtin_bit_cast(bf16x8_t, u32x4_t{pa[0], pa[1], pb[0], pb[1]});
      const bf16x8_t pl = __builtin_bit_cast(bf16x8_t, u32x4_t{pa[2], pa[3], pb[2], pb[3]});
      bf16x8_t vf[CT];
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        const unsigned char* vp = tile + vaddr[t] + s * (32 * R * 2);
        const s16x4_t va = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)(vp));
        const s16x4_t vb = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4_t __attribute__((address_space(3)))*)(vp + 16 * R * 2));
        typedef __attribute__((ext_vector_type(8))) short s16x8_t;
        const s16x8_t vv = {va[0], va[1], va[2], va[3], vb[0], vb[1], vb[2], vb[3]};
        vf[t] = __builtin_bit_cast(bf16x8_t, vv);
      }
#pragma unroll
      for (int t = 0; t < CT; ++t) o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[t], pl, o[t], 0, 0, 0);
#pragma unroll
      for (int t = 0; t < CT; ++t) o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[t], ph, o[t], 0, 0, 0);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (g == 0) s_sum[ht][w4][fr] = l;
  __syncthreads();
  if (h0 + fr >= H) return;
  const long long slot = (static_cast<long long>(b) * H + h0 + fr) * nsplit + split;
#pragma unroll
  for (int t = 0; t < CT; ++t) *reinterpret_cast<f32x4_t*>(part_o + slot * R + (w4 * CT + t) * 16 + g * 4) = o[t];
  if (w4 == 0 && g == 0) {
    part_ml[slot * 2] = m * scale_log2e;
    part_ml[slot * 2 + 1] = s_sum[ht][0][fr] + s_sum[ht][1][fr] + s_sum[ht][2][fr] + s_sum[ht][3][fr];
  }
}
template <int R, int HT>
static void launch_attend(const bf16_t* q, const bf16_t* cache, float* part_o, float* part_ml, const int* row_slot,
                          const int* pos, int rows, int H, int cap, int nsplit, float scale, hipStream_t st) {
  constexpr int lds = 2 * LT_KEYS * R * 2 + HT * 4096;
  static const bool attr = [] {
    return hipFuncSetAttribute(reinterpret_cast<const void*>(latent_attend_kernel<R, HT>),
                               hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
  }();
  (void)attr;
  hipLaunchKernelGGL((latent_attend_kernel<R, HT>), dim3(nsplit, rows, (H + 16 * HT - 1) / (16 * HT)), dim3(256 * HT), lds, st, q, cache,
                     part_o, part_ml, row_slot, pos, H, cap, scale * 1.4426950408889634f);
}
void launch_latent_attend(const bf16_t* q, const bf16_t* cache, float* part_o, float* part_ml, const int* row_slot,
                          const int* pos, int rows, int H, int R, int cap, int nsplit, float scale, hipStream_t st) {
#define EVGPT_ATTEND(R_)                                                                                        \
  if (H > 16) launch_attend<R_, 2>(q, cache, part_o, part_ml, row_slot, pos, rows, H, cap, nsplit, scale, st);  \
  else launch_attend<R_, 1>(q, cache, part_o, part_ml, row_slot, pos, rows, H, cap, nsplit, scale, st)
  if (R == 64) { EVGPT_ATTEND(64); }
  else if (R == 128) { EVGPT_ATTEND(128); }
  else if (R == 256) { EVGPT_ATTEND(256); }
  else if (R == 384) { EVGPT_ATTEND(384); }
  else { EVGPT_ATTEND(512); }
#undef EVGPT_ATTEND
}

}  // namespace evgpt
