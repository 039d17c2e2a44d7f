// Weight-streaming products of up to four rows with an fp32 residual stream: y = epilogue(W · input(x)).
//
// A block is four waves on one unit of four output rows: each wave streams a quarter of the contraction
// (16-byte non-temporal loads, the next batch in flight while the current one is multiplied), the partial sums
// meet in LDS.  Blocks walk the units, and the first unit's weights are requested before the block prepares its
// input, which it keeps in LDS in the storage type:
//   NORM   norm (RMS or layer norm) of the stream;
//   MERGE  x + (rms(a) wa + rms(b) wb) / 2, its RMS norm, and (one block) the new stream;
//   POST   x + norm(a) wa, its norm, and (one block) the new stream;
//   ROWS   RMS norm of a run of columns of a projection's rows;
//   GROUP  group norm of a recurrent mixer's output, with a sigmoid gate after it if asked for;
//   PLAIN  a row that is already in the storage type, read from global memory.
// Epilogues store fp32 rows (scaled and softly capped if asked for), add to the stream, or multiply gate and up
// rows (GLU).  Two problems with the same epilogue (the output projections of two branches) can share a launch.  One more
// block can norm another run of columns into a latent cache.
#include "src_rows.h"

namespace evgpt {

constexpr int GV_R = 4;        // output rows per unit
constexpr int GV_NI = 2;       // 16-byte chunks per thread and row in a batch

__device__ __forceinline__ float dot16(const u32x4_t& w, const u32x4_t& x, float acc, bf16_t) { return dot8_bf16(w, x, acc); }
__device__ __forceinline__ float dot16(const u32x4_t& w, const u32x4_t& x, float acc, float) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc += __uint_as_float(w[i]) * __uint_as_float(x[i]);
  return acc;
}

constexpr int GV_KEEP = 2;     // chunks of eight a thread keeps while it norms a row (4096 columns)

// f(k, c) for the thread's kept chunks of a row of K columns
template <typename F> __device__ __forceinline__ void kept_chunks(int K, F f) {
#pragma unroll
  for (int k = 0; k < GV_KEEP; ++k) {
    const int c = (threadIdx.x + k * 256) * 8;
    if (c < K) f(k, c);
  }
}

// ALL: either norm, the stream or columns of a projection; otherwise the RMS norm of the stream
template <typename T, bool ALL>
__device__ void prepare_norm(const GemvInput& in, int b, int K, T* xs, float* red, bool lead) {
  const float* x = static_cast<const float*>(in.x) + static_cast<long long>(b) * K;
  const bool rows = ALL && in.kind == GV_ROWS;
  float keep[GV_KEEP][8], wk[GV_KEEP][8];
  auto value = [&](int c, float (&v)[8]) {
    if (!rows) load8(x + c, v);
    else section8(in.gate, b, in.gcol, in.n, c, v);
  };
  kept_chunks(K, [&](int k, int c) { value(c, keep[k]); load8(in.w + c, wk[k]); });
  const RowStat st = row_stat<GV_KEEP>(keep, in.n, K, in.eps, ALL && in.layer != 0, red, value);
  auto put = [&](int c, const float (&v)[8], float (&w)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) w[i] *= (v[i] - st.mean) * st.r;
    store8(xs + c, w);
    if (ALL && lead && in.xn_out) store8(static_cast<T*>(in.xn_out) + static_cast<long long>(b) * K + c, w);
  };
  kept_chunks(K, [&](int k, int c) { put(c, keep[k], wk[k]); });
  for (int c = (threadIdx.x + GV_KEEP * 256) * 8; c < K; c += 2048) {
    float v[8], w[8];
    value(c, v);
    load8(in.w + c, w);
    put(c, v, w);
  }
}

// (every operand of the kept chunks is requested before the first sum)
template <typename T>
__device__ void prepare_post(const GemvInput& in, int b, int K, T* xs, float* red, bool lead) {
  const long long o = static_cast<long long>(b) * K;
  const float* x = static_cast<const float*>(in.x) + o;
  float keep[GV_KEEP][8], xk[GV_KEEP][8], ak[GV_KEEP][8], wk[GV_KEEP][8];
  auto branch = [&](int c, float (&v)[8]) { load8(in.a + o + c, v); };
  kept_chunks(K, [&](int k, int c) { branch(c, keep[k]); load8(x + c, xk[k]); load8(in.wa + c, ak[k]); load8(in.w + c, wk[k]); });
  const RowStat sa = row_stat<GV_KEEP>(keep, in.n, K, in.eps, in.layer != 0, red, branch);
  auto add = [&](float (&v)[8], const float (&u)[8], const float (&p)[8]) {           // branch values -> the new stream
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = u[i] + (v[i] - sa.mean) * sa.r * p[i];
  };
  auto value = [&](int c, float (&v)[8]) {
    float u[8], p[8];
    branch(c, v);
    load8(x + c, u);
    load8(in.wa + c, p);
    add(v, u, p);
  };
  kept_chunks(K, [&](int k, int) { add(keep[k], xk[k], ak[k]); });
  const RowStat st = row_stat<GV_KEEP>(keep, in.n, K, in.eps, in.layer != 0, red, value);
  auto put = [&](int c, const float (&v)[8], float (&w)[8]) {
    if (lead) store8(in.x_out + o + c, v);
#pragma unroll
    for (int i = 0; i < 8; ++i) w[i] *= (v[i] - st.mean) * st.r;
    store8(xs + c, w);
    if (lead && in.xn_out) store8(static_cast<T*>(in.xn_out) + o + c, w);
  };
  kept_chunks(K, [&](int k, int c) { put(c, keep[k], wk[k]); });
  for (int c = (threadIdx.x + GV_KEEP * 256) * 8; c < K; c += 2048) {
    float v[8], w[8];
    value(c, v);
    load8(in.w + c, w);
    put(c, v, w);
  }
}

// The block past the units: RMS norm of the latent columns of every row into the row's cache, a wave per row.
template <typename T>
__device__ void store_latents(const LatentStore& s, int B) {
  const int lane = threadIdx.x & 63;
  for (int b = threadIdx.x >> 6; b < B; b += 4) {
    if (s.live && !s.live[b]) continue;
    const int p = min(max(s.pos[b], 0), s.cap - 1);
    latent_row(s.src, b, s.col, s.n, s.R, s.w, s.eps, static_cast<T*>(s.cache) + (static_cast<long long>(b) * s.cap + p) * s.R, lane);
  }
}

template <typename T>
__device__ void prepare_merge(const GemvInput& in, int b, int K, T* xs, float* red, bool lead) {
  const long long o = static_cast<long long>(b) * K;
  const float* x = static_cast<const float*>(in.x) + o;
  float sa = 0.f, sb = 0.f;
  for (int c = threadIdx.x * 8; c < K; c += 2048) {
    float v[8];
    load8(in.a + o + c, v);
    sa += sumsq8(v);
    load8(in.b + o + c, v);
    sb += sumsq8(v);
  }
  const float inv_n = 1.f / static_cast<float>(in.n);
  const float ra = 0.5f * rsqrtf(block_sum(sa, red) * inv_n + in.eps);
  const float rb = 0.5f * rsqrtf(block_sum(sb, red) * inv_n + in.eps);
  float ss = 0.f;
  auto value = [&](int c, float (&v)[8]) {
    float p[8], q[8];
    load8(x + c, v);
    load8(in.a + o + c, p);
    load8(in.wa + c, q);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] += p[i] * ra * q[i];
    load8(in.b + o + c, p);
    load8(in.wb + c, q);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] += p[i] * rb * q[i];
  };
  for (int c = threadIdx.x * 8; c < K; c += 2048) {
    float v[8];
    value(c, v);
    ss += sumsq8(v);
    if (lead) store8(in.x_out + o + c, v);
  }
  const float r = rsqrtf(block_sum(ss, red) * inv_n + in.eps);
  for (int c = threadIdx.x * 8; c < K; c += 2048) {
    float v[8], w[8];
    value(c, v);
    load8(in.w + c, w);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= r * w[i];
    store8(xs + c, v);
  }
}

template <typename T>
__device__ void prepare_group(const GemvInput& in, int b, int K, T* xs, float* inv) {
  const int slots = in.heads * in.vp, plen = in.heads * in.v / in.parts;
  const float* y = in.y + static_cast<long long>(b) * slots;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  __syncthreads();                      // inv of the row before
  const bool dense = in.v == in.vp && (plen & 7) == 0;
  for (int p = wid; p < in.parts; p += 4) {
    float s = 0.f;
    if (dense) {
      for (int i = lane * 8; i < plen; i += 512) {
        float t[8];
        load8(y + p * plen + i, t);
        s += sumsq8(t);
      }
    } else {
      for (int i = lane; i < plen; i += 64) {
        const int c = p * plen + i;
        const float t = y[(c / in.v) * in.vp + c % in.v];
        s += t * t;
      }
    }
    s = wave_sum(s);
    if (lane == 0) inv[p] = rsqrtf(s / static_cast<float>(plen) + in.eps);
  }
  __syncthreads();
  for (int c = threadIdx.x * 8; c < K; c += 2048) {
    float a[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    if (c < slots) {
      float w[8];
      load8(y + c, a);
      load8(in.w + c, w);
      const int h = c / in.vp, c0 = h * in.v + c % in.vp;
      const int part0 = min(c0 / plen, in.parts - 1), next = (part0 + 1) * plen;
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] *= inv[c0 + i < next ? part0 : min((c0 + i) / plen, in.parts - 1)] * w[i];
      if (in.gate_mode == GATE_SIGMOID_AFTER) {
        float t[8];
        src8(in.gate, b, in.gcol + c, t);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] *= sigmoid_f(t[i]);
      }
    }
    store8(xs + c, a);
  }
}

// PREP_NONE: every problem reads its input rows from global memory; otherwise all are staged (PLAIN rows copied): PREP_RMS for
// the RMS norm of the stream, branches and group norms, PREP_ALL for either norm of the stream, the norm after a
// sublayer and columns of a projection, with the latent store and the finished rows.
enum { PREP_NONE = 0, PREP_RMS = 1, PREP_ALL = 2 };
template <typename T, int B, int EPI, int PREP>
__global__ __launch_bounds__(256) void row_gemv_kernel(GemvCall call, int blocks0) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  constexpr int CE = 16 / sizeof(T);                      // elements per 16-byte chunk
  __shared__ float part[2][4][GV_R * B];
  __shared__ float red[16];
  constexpr bool PLAIN = PREP == PREP_NONE;
  if constexpr (PREP == PREP_ALL) {
    if (call.latent.cache && blockIdx.x + 1 == gridDim.x) {
      store_latents<T>(call.latent, B);
      return;
    }
  }
  const bool second = call.count == 2 && static_cast<int>(blockIdx.x) >= blocks0;
  const GemvProblem& p = call.p[second ? 1 : 0];
  const int blk = second ? blockIdx.x - blocks0 : blockIdx.x;
  const int nblk = call.count == 2 ? (second ? gridDim.x - blocks0 : blocks0) : blocks0;
  const int K = p.K, nchunk = K / CE, nit = (nchunk + 255) / 256;
  const int units = EPI == GV_GLU ? p.N / 4 : p.N / GV_R;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const T* W = static_cast<const T*>(p.W);
  T* xs = reinterpret_cast<T*>(smem);
  auto row_of = [&](int u, int r) {       // GLU: two gate rows, then the matching up rows
    return EPI == GV_GLU ? (r < 2 ? u * 2 + r : p.N / 2 + u * 2 + r - 2) : u * GV_R + r;
  };
  u32x4_t cur[GV_NI][GV_R], nxt[GV_NI][GV_R];
  auto fetch = [&](u32x4_t (&w)[GV_NI][GV_R], int u, int it) {
#pragma unroll
    for (int i = 0; i < GV_NI; ++i) {
      const int ch = (it + i) * 256 + tid;
      if (ch < nchunk) {
#pragma unroll
        for (int r = 0; r < GV_R; ++r) w[i][r] = load_stream16(W + static_cast<long long>(row_of(u, r)) * K + ch * CE);
      }
    }
  };
  if (blk < units) fetch(cur, blk, 0);
  if constexpr (!PLAIN) {
    for (int b = 0; b < B; ++b) {
      T* xb = xs + static_cast<long long>(b) * K;
      if constexpr (PREP == PREP_ALL) {
        if (p.in.kind == GV_POST) prepare_post(p.in, b, K, xb, red, blk == 0);
        else prepare_norm<T, true>(p.in, b, K, xb, red, blk == 0);
      } else if (p.in.kind == GV_NORM) prepare_norm<T, false>(p.in, b, K, xb, red, blk == 0);
      else if (p.in.kind == GV_MERGE) prepare_merge(p.in, b, K, xb, red, blk == 0);
      else if (p.in.kind == GV_GROUP) prepare_group(p.in, b, K, xb, reinterpret_cast<float*>(smem + static_cast<long long>(B) * K * sizeof(T)));
      else
        for (int c = tid; c < nchunk; c += 256)
          reinterpret_cast<u32x4_t*>(xb)[c] = load16(static_cast<const T*>(p.in.x) + static_cast<long long>(b) * K + c * CE);
    }
    __syncthreads();
  }
  const T* xg = static_cast<const T*>(p.in.x);
  int flip = 0;
  for (int u = blk; u < units; u += nblk) {
    float acc[GV_R][B];
#pragma unroll
    for (int r = 0; r < GV_R; ++r)
#pragma unroll
      for (int b = 0; b < B; ++b) acc[r][b] = 0.f;
    for (int it = 0; it < nit; it += GV_NI) {
      if (it + GV_NI < nit) fetch(nxt, u, it + GV_NI);
      else if (u + nblk < units) fetch(nxt, u + nblk, 0);
#pragma unroll
      for (int i = 0; i < GV_NI; ++i) {
        const int ch = (it + i) * 256 + tid;
        if (ch < nchunk) {
#pragma unroll
          for (int b = 0; b < B; ++b) {
            u32x4_t x;
            if constexpr (PLAIN) x = load16(xg + static_cast<long long>(b) * K + ch * CE);
            else x = *reinterpret_cast<const u32x4_t*>(xs + static_cast<long long>(b) * K + ch * CE);
#pragma unroll
            for (int r = 0; r < GV_R; ++r) acc[r][b] = dot16(cur[i][r], x, acc[r][b], T(0));
          }
        }
      }
#pragma unroll
      for (int i = 0; i < GV_NI; ++i)
#pragma unroll
        for (int r = 0; r < GV_R; ++r) cur[i][r] = nxt[i][r];
    }
#pragma unroll
    for (int r = 0; r < GV_R; ++r)
#pragma unroll
      for (int b = 0; b < B; ++b) {
        const float s = wave_sum(acc[r][b]);
        if (lane == 0) part[flip][wid][r * B + b] = s;
      }
    __syncthreads();
    auto total = [&](int i) { return part[flip][0][i] + part[flip][1][i] + part[flip][2][i] + part[flip][3][i]; };
    if constexpr (EPI == GV_GLU) {
      if (tid < 2 * B) {
        const int r = tid / B, b = tid % B;
        const float g = total(r * B + b), v = total((r + 2) * B + b);
        static_cast<T*>(call.h)[static_cast<long long>(b) * (p.N / 2) + u * 2 + r] =
            from_f32<T>((call.act == GLU_SILU ? g * sigmoid_f(g) : gelu_tanh_f(g)) * v);
      }
    } else {
      if (tid < GV_R * B) {
        const int r = tid / B, b = tid % B;
        float* y = p.y + static_cast<long long>(b) * p.ldy + u * GV_R + r;
        if constexpr (EPI == GV_ADD) *y += total(r * B + b);
        else *y = PREP == PREP_ALL && call.finish ? soft_cap(total(r * B + b), call.scale, call.cap) : total(r * B + b);
      }
    }
    flip ^= 1;       // the next unit's partial sums go to the other buffer: one barrier per unit
  }
}

static int g_blocks = 0;
void row_gemv_blocks(int n) { g_blocks = n > 0 ? n : 0; }

static int blocks_of(const GemvProblem& p, int budget) {
  const int units = p.N / GV_R;
  return units < budget ? units : budget;
}
size_t row_gemv_lds(const GemvCall& c, bool f32, int B) {
  size_t most = 0;
  for (int i = 0; i < c.count; ++i) {
    const GemvInput& in = c.p[i].in;
    if (in.kind == GV_PLAIN && c.count == 1) continue;
    const size_t need = static_cast<size_t>(B) * c.p[i].K * (f32 ? 4 : 2) + (in.kind == GV_GROUP ? in.parts * 4 : 0);
    most = need > most ? need : most;
  }
  return most;
}
template <typename T, int B>
static void launch_b(const GemvCall& c, size_t lds, hipStream_t st) {
  // two or three blocks per CU: enough waves to stream, few enough that the inputs are not prepared too often.  Width 4096,
  // us at 256 / 512 / 768 / 1280 / 2048 blocks: one row, norm + 18560 rows 38.5 / 26.5 / 26.8 / 28.9 / 29.9, merge + gate/up
  // 45.8 / 33.4 / 35.4 / 40.2 / 42.0, two output projections 19.8 / 18.3 / 15.9 / 18.0 / 21.3; four rows, norm + 18560 rows
  // 58.9 / 38.8 / 34.6 / 41.6 / 47.4
  const int kind = c.p[0].in.kind;
  const int budget = g_blocks ? g_blocks : (B == 1 && c.count == 1 && (kind == GV_NORM || kind == GV_MERGE || kind == GV_POST) ? 512 : 768);
  const int b0 = blocks_of(c.p[0], c.count == 2 ? budget / 2 : budget), b1 = c.count == 2 ? blocks_of(c.p[1], budget / 2) : 0;
  const dim3 grid(b0 + b1 + (c.latent.cache ? 1 : 0)), block(256);
  const bool plain = c.count == 1 && kind == GV_PLAIN;
  const bool all = c.count == 1 && (kind == GV_POST || kind == GV_ROWS || (kind == GV_NORM && (c.p[0].in.layer || c.p[0].in.xn_out || c.finish)));
#define EVGPT_GEMV(E)                                                                                    \
  if (plain) hipLaunchKernelGGL((row_gemv_kernel<T, B, E, PREP_NONE>), grid, block, 0, st, c, b0);       \
  else hipLaunchKernelGGL((row_gemv_kernel<T, B, E, PREP_RMS>), grid, block, lds, st, c, b0)
  // (nothing is added to the stream behind a PREP_ALL input)
  if (all && c.epilogue == GV_GLU) hipLaunchKernelGGL((row_gemv_kernel<T, B, GV_GLU, PREP_ALL>), grid, block, lds, st, c, b0);
  else if (all) hipLaunchKernelGGL((row_gemv_kernel<T, B, GV_STORE, PREP_ALL>), grid, block, lds, st, c, b0);
  else if (c.epilogue == GV_STORE) { EVGPT_GEMV(GV_STORE); }
  else if (c.epilogue == GV_ADD) { EVGPT_GEMV(GV_ADD); }
  else { EVGPT_GEMV(GV_GLU); }
#undef EVGPT_GEMV
}
void launch_row_gemv(const GemvCall& c, bool f32, int B, hipStream_t st) {
  const size_t lds = row_gemv_lds(c, f32, B);
  if (f32) {
    if (B == 1) launch_b<float, 1>(c, lds, st);
    else if (B == 2) launch_b<float, 2>(c, lds, st);
    else if (B == 3) launch_b<float, 3>(c, lds, st);
    else launch_b<float, 4>(c, lds, st);
  } else {
    if (B == 1) launch_b<bf16_t, 1>(c, lds, st);
    else if (B == 2) launch_b<bf16_t, 2>(c, lds, st);
    else if (B == 3) launch_b<bf16_t, 3>(c, lds, st);
    else launch_b<bf16_t, 4>(c, lds, st);
  }
}

}  // namespace evgpt
