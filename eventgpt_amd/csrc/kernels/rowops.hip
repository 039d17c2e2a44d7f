// Row kernels around the projections of a layered decoder: the residual stream x is fp32, every norm,
// gate and rotation is fp32, and what a projection reads is written in the storage type T.
//
// One block per row.  A row of a projection (`SrcRows`) may still be split-K slabs, which are summed on
// load.  Row widths are padded to multiples of 64 by zeros (weights are padded when they are packed), so
// all accesses are aligned vectors; norms divide by the true width.
#include "src_rows.h"

namespace evgpt {

template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(const int* __restrict__ tok, const T* __restrict__ embed,
                                                         float scale, float* __restrict__ x, int ld, int vocab) {
  const long long row = blockIdx.x;
  int t = tok[row];
  if (t < 0 || t >= vocab) t = 0;
  for (int c = threadIdx.x * 8; c < ld; c += 2048) {
    float v[8];
    load8(embed + static_cast<long long>(t) * ld + c, v);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= scale;
    store8(x + row * ld + c, v);
  }
}
void launch_embed_rows(const int* tok, const void* embed, bool f32, float scale, float* x, int rows, int ld, int vocab,
                       hipStream_t st) {
  if (f32)
    hipLaunchKernelGGL(embed_rows_kernel<float>, dim3(rows), dim3(256), 0, st, tok, static_cast<const float*>(embed),
                       scale, x, ld, vocab);
  else
    hipLaunchKernelGGL(embed_rows_kernel<bf16_t>, dim3(rows), dim3(256), 0, st, tok,
                       static_cast<const bf16_t*>(embed), scale, x, ld, vocab);
}

// The residual kernels.  MODE 0: xn = norm(x).  MODE 1: x += a first.  MODE 2: x += (norm(a) wa + norm(b) wb) / 2
// first.  MODE 3: x += norm(a) wa first.  MODE 4: the same (or x += y without wa) with y the weighted sum of a few
// rows of another matrix.  norm: RMS, or layer norm (LN).  A thread keeps its first NC chunks of eight in registers
// between the passes; MODE 3 and 4 request the stream and the branch's weights with the branch.
template <typename T, int MODE, bool LN, int NC>
__global__ __launch_bounds__(256) void residual_norm_kernel(float* __restrict__ x, const int* __restrict__ sel,
                                                            SrcRows a, SrcRows b, MixRows mix, const float* __restrict__ wa,
                                                            const float* __restrict__ wb, const float* __restrict__ w,
                                                            T* __restrict__ xn, int n, int ld, float eps) {
  __shared__ float red[16];
  const long long row = blockIdx.x, xrow = MODE == 0 && sel ? sel[row] : row;
  float* xr = x + xrow * ld;
  float keep[NC][8];
  constexpr int NX = MODE >= 3 ? NC : 1;
  float xk[NX][8], ak[NX][8];
  float ra = 0.f, rb = 0.f;
  RowStat sy{0.f, 1.f};
  auto branch = [&](int c, float (&v)[8]) {          // MODE 3 and 4: the sublayer's output
    if constexpr (MODE == 3) src8(a, row, c, v);
    if constexpr (MODE == 4) {
      const int* pick = mix.pick + row * mix.top;
      const float* pw = mix.w + row * mix.top;
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = 0.f;
      for (int k = 0; k < mix.top; ++k) {
        float t[8];
        load8(static_cast<const T*>(mix.y) + static_cast<long long>(pick[k]) * mix.ld + c, t);
        const float f = pw[k];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] += f * t[i];
      }
    }
  };
  if constexpr (MODE == 2) {
    const float inv_n = 1.f / static_cast<float>(n);
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x * 8; c < ld; c += 2048) {
      float t[8];
      src8(a, row, c, t);
      sa += sumsq8(t);
      src8(b, row, c, t);
      sb += sumsq8(t);
    }
    ra = 0.5f * rsqrtf(block_sum(sa, red) * inv_n + eps);
    rb = 0.5f * rsqrtf(block_sum(sb, red) * inv_n + eps);
  }
  if constexpr (MODE >= 3) {
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (threadIdx.x + k * 256) * 8;
      if (c < ld) {
        branch(c, keep[k]);
        load8(xr + c, xk[k]);
        if (MODE == 3 || wa) load8(wa + c, ak[k]);       // (zero in the padding)
      }
    }
    if (MODE == 3 || wa) sy = row_stat<NC>(keep, n, ld, eps, LN, red, branch);
  }
  auto post = [&](float (&v)[8], const float (&u)[8], const float (&p)[8]) {       // branch values -> the new stream
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = MODE == 3 || wa ? u[i] + (v[i] - sy.mean) * sy.r * p[i] : u[i] + v[i];
  };
  auto value = [&](int c, float (&v)[8]) {
    load8(xr + c, v);
    if constexpr (MODE == 1) {
      float t[8];
      src8(a, row, c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] += t[i];
    }
    if constexpr (MODE == 2) {
      float t[8], u[8], p[8], q[8];
      src8(a, row, c, t);
      src8(b, row, c, u);
      load8(wa + c, p);
      load8(wb + c, q);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] += t[i] * ra * p[i] + u[i] * rb * q[i];
    }
    if constexpr (MODE != 0) store8(xr + c, v);
  };
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (threadIdx.x + k * 256) * 8;
    if (c >= ld) continue;
    if constexpr (MODE >= 3) {
      post(keep[k], xk[k], ak[k]);
      store8(xr + c, keep[k]);
    } else {
      value(c, keep[k]);
    }
  }
  if constexpr (MODE != 0)
    for (int c = (threadIdx.x + NC * 256) * 8; c < ld; c += 2048) {
      float v[8];
      if constexpr (MODE >= 3) {
        float u[8], p[8];
        branch(c, v);
        load8(xr + c, u);
        if (MODE == 3 || wa) load8(wa + c, p);
        post(v, u, p);
        store8(xr + c, v);
      } else {
        value(c, v);
      }
    }
  if (w == nullptr) return;
  // each thread re-reads what it wrote
  const RowStat st = row_stat<NC>(keep, n, ld, eps, LN, red, [&](int c, float (&v)[8]) { load8(xr + c, v); });
  T* o = xn + row * ld;
  auto put = [&](int c, const float (&v)[8]) {
    float g[8];
    load8(w + c, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) g[i] *= (v[i] - st.mean) * st.r;
    store8(o + c, g);
  };
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (threadIdx.x + k * 256) * 8;
    if (c < ld) put(c, keep[k]);
  }
  for (int c = (threadIdx.x + NC * 256) * 8; c < ld; c += 2048) {
    float v[8];
    load8(xr + c, v);
    put(c, v);
  }
}
template <int MODE>
static void launch_residual(float* x, const int* sel, const SrcRows& a, const SrcRows& b, const MixRows& mix, const float* wa,
                            const float* wb, const float* w, void* xn, bool f32, int rows, int n, int ld, float eps,
                            bool layer, hipStream_t st) {
#define EVGPT_RES(T, LN) \
  if (ld <= 4096) hipLaunchKernelGGL((residual_norm_kernel<T, MODE, LN, 2>), dim3(rows), dim3(256), 0, st, x, sel, a, b, mix, wa, wb, w, \
                                     static_cast<T*>(xn), n, ld, eps); \
  else hipLaunchKernelGGL((residual_norm_kernel<T, MODE, LN, 4>), dim3(rows), dim3(256), 0, st, x, sel, a, b, mix, wa, wb, w, \
                          static_cast<T*>(xn), n, ld, eps)
  if (layer) { if (f32) { EVGPT_RES(float, true); } else { EVGPT_RES(bf16_t, true); } }
  else { if (f32) { EVGPT_RES(float, false); } else { EVGPT_RES(bf16_t, false); } }
#undef EVGPT_RES
}
void launch_norm_rows(const float* x, const int* sel, const float* w, void* xn, bool f32, int rows, int n, int ld,
                      float eps, bool layer, hipStream_t st) {
  launch_residual<0>(const_cast<float*>(x), sel, SrcRows{}, SrcRows{}, MixRows{}, nullptr, nullptr, w, xn, f32, rows, n, ld, eps, layer, st);
}
void launch_add_norm_rows(float* x, const SrcRows& y, const float* w, void* xn, bool f32, int rows, int n, int ld,
                          float eps, bool layer, hipStream_t st) {
  launch_residual<1>(x, nullptr, y, SrcRows{}, MixRows{}, nullptr, nullptr, w, xn, f32, rows, n, ld, eps, layer, st);
}
void launch_merge_norm_rows(float* x, const SrcRows& a, const SrcRows& b, const float* wa, const float* wb,
                            const float* w, void* xn, bool f32, int rows, int n, int ld, float eps, hipStream_t st) {
  launch_residual<2>(x, nullptr, a, b, MixRows{}, wa, wb, w, xn, f32, rows, n, ld, eps, false, st);
}
void launch_post_norm_rows(float* x, const SrcRows& y, const float* wy, const float* w, void* xn, bool f32, int rows, int n,
                           int ld, float eps, bool layer, hipStream_t st) {
  launch_residual<3>(x, nullptr, y, SrcRows{}, MixRows{}, wy, nullptr, w, xn, f32, rows, n, ld, eps, layer, st);
}
void launch_mix_norm_rows(float* x, const MixRows& y, const float* wy, const float* w, void* xn, bool f32, int rows, int n,
                          int ld, float eps, bool layer, hipStream_t st) {
  launch_residual<4>(x, nullptr, SrcRows{}, SrcRows{}, y, wy, nullptr, w, xn, f32, rows, n, ld, eps, layer, st);
}

// logits = cap * tanh(scale * logits / cap); cap 0: scale alone
__global__ __launch_bounds__(256) void cap_logits_kernel(float* __restrict__ x, long long n, float scale, float cap) {
  for (long long i = (blockIdx.x * 256ll + threadIdx.x) * 4; i < n; i += gridDim.x * 1024ll) {
    f32x4_t v = load4(x + i);
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = soft_cap(v[k], scale, cap);
    *reinterpret_cast<f32x4_t*>(x + i) = v;
  }
}
void launch_cap_logits(float* x, long long n, float scale, float cap, hipStream_t st) {
  const long long want = (n + 1023) / 1024;
  hipLaunchKernelGGL(cap_logits_kernel, dim3(static_cast<unsigned>(want < 4096 ? want : 4096)), dim3(256), 0, st, x, n, scale, cap);
}

template <typename T, int ACT>
__global__ __launch_bounds__(256) void glu_rows_kernel(SrcRows src, T* __restrict__ h, long long total, int ip) {
  const int per = ip >> 3;
  for (long long i = blockIdx.x * 256ll + threadIdx.x; i < total; i += gridDim.x * 256ll) {
    const long long row = i / per;
    const int c = static_cast<int>(i % per) * 8;
    float a[8], b[8];
    src8(src, row, c, a);
    src8(src, row, ip + c, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] = (ACT == GLU_SILU ? a[j] * sigmoid_f(a[j]) : gelu_tanh_f(a[j])) * b[j];
    store8(h + row * ip + c, a);
  }
}
void launch_glu_rows(const SrcRows& src, void* h, bool f32, int rows, int ip, int act, hipStream_t st) {
  const long long total = static_cast<long long>(rows) * (ip / 8);
  const long long want = (total + 255) / 256;
  const dim3 grid(static_cast<unsigned>(want < 4096 ? want : 4096)), block(256);
  if (f32) {
    if (act == GLU_SILU) hipLaunchKernelGGL((glu_rows_kernel<float, GLU_SILU>), grid, block, 0, st, src, static_cast<float*>(h), total, ip);
    else hipLaunchKernelGGL((glu_rows_kernel<float, GLU_GELU_TANH>), grid, block, 0, st, src, static_cast<float*>(h), total, ip);
  } else {
    if (act == GLU_SILU) hipLaunchKernelGGL((glu_rows_kernel<bf16_t, GLU_SILU>), grid, block, 0, st, src, static_cast<bf16_t*>(h), total, ip);
    else hipLaunchKernelGGL((glu_rows_kernel<bf16_t, GLU_GELU_TANH>), grid, block, 0, st, src, static_cast<bf16_t*>(h), total, ip);
  }
}

// Group norm with a gate.  The row is staged in LDS (gated first when the gate comes before the norm), every
// part's root mean square is taken over its run of true channels -- a wave per part -- and the row is written
// with the part of each channel looked up.
template <typename T, int GATE>
__global__ __launch_bounds__(256) void group_norm_kernel(SrcRows y, SrcRows gate, int gcol,
                                                         const float* __restrict__ w, T* __restrict__ out, int heads,
                                                         int v, int vp, int parts, int ld_out, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row_lds[];   // [heads * vp] values, then [parts]
  const int slots = heads * vp, plen = heads * v / parts;
  float* inv = row_lds + slots;
  const long long row = blockIdx.x;
  for (int c = threadIdx.x * 8; c < slots; c += 2048) {
    float a[8];
    src8(y, row, c, a);
    if constexpr (GATE == GATE_SILU_BEFORE) {
      float g[8];
      src8(gate, row, gcol + c, g);
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] *= g[i] * sigmoid_f(g[i]);
    }
    store8(row_lds + c, a);
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  if (v == vp && (plen & 7) == 0 && parts >= 4) {      // no padding between heads: a part is a run of the row
    for (int p = wid; p < parts; p += 4) {
      float s = 0.f;
      for (int i = lane * 8; i < plen; i += 512) {
        float t[8];
        load8(row_lds + p * plen + i, t);
        s += sumsq8(t);
      }
      s = wave_sum(s);
      if (lane == 0) inv[p] = rsqrtf(s / static_cast<float>(plen) + eps);
    }
  } else if (parts >= 4) {
    for (int p = wid; p < parts; p += 4) {
      float s = 0.f;
      for (int i = lane; i < plen; i += 64) {
        const int c = p * plen + i;
        const float t = row_lds[(c / v) * vp + c % v];
        s += t * t;
      }
      s = wave_sum(s);
      if (lane == 0) inv[p] = rsqrtf(s / static_cast<float>(plen) + eps);
    }
  } else {
    __shared__ float red[16];
    for (int p = 0; p < parts; ++p) {
      float s = 0.f;
      for (int i = threadIdx.x; i < plen; i += 256) {
        const int c = p * plen + i;
        const float t = row_lds[(c / v) * vp + c % v];
        s += t * t;
      }
      s = block_sum(s, red);
      if (threadIdx.x == 0) inv[p] = rsqrtf(s / static_cast<float>(plen) + eps);
    }
  }
  __syncthreads();
  for (int c = threadIdx.x * 8; c < ld_out; c += 2048) {
    float a[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    if (c < slots) {
      float g[8];
      load8(row_lds + c, a);
      load8(w + c, g);
      const int h = c / vp, c0 = h * v + c % vp;      // vp is a multiple of 8: eight slots of one head
      const int part0 = min(c0 / plen, parts - 1), next = (part0 + 1) * plen;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        // (padding slots have zero weight)
        const int part = c0 + i < next ? part0 : min((c0 + i) / plen, parts - 1);
        a[i] *= inv[part] * g[i];
      }
      if constexpr (GATE == GATE_SIGMOID_AFTER) {
        float t[8];
        src8(gate, row, gcol + c, t);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] *= sigmoid_f(t[i]);
      }
    }
    store8(out + row * ld_out + c, a);
  }
}
template <typename T>
static void launch_group_norm(const SrcRows& y, const SrcRows& gate, int gcol, int mode, const float* w, void* out, int rows,
                              int heads, int v, int vp, int parts, int ld_out, float eps, hipStream_t st) {
  const size_t lds = (static_cast<size_t>(heads) * vp + parts) * 4;
  const dim3 grid(rows), block(256);
  T* o = static_cast<T*>(out);
  if (lds > 64 * 1024)
    hipFuncSetAttribute(mode == GATE_SILU_BEFORE ? reinterpret_cast<const void*>(&group_norm_kernel<T, GATE_SILU_BEFORE>)
                        : mode == GATE_SIGMOID_AFTER ? reinterpret_cast<const void*>(&group_norm_kernel<T, GATE_SIGMOID_AFTER>)
                                                     : reinterpret_cast<const void*>(&group_norm_kernel<T, GATE_NONE>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds));
  if (mode == GATE_SILU_BEFORE)
    hipLaunchKernelGGL((group_norm_kernel<T, GATE_SILU_BEFORE>), grid, block, lds, st, y, gate, gcol, w, o, heads, v, vp, parts, ld_out, eps);
  else if (mode == GATE_SIGMOID_AFTER)
    hipLaunchKernelGGL((group_norm_kernel<T, GATE_SIGMOID_AFTER>), grid, block, lds, st, y, gate, gcol, w, o, heads, v, vp, parts, ld_out, eps);
  else
    hipLaunchKernelGGL((group_norm_kernel<T, GATE_NONE>), grid, block, lds, st, y, gate, gcol, w, o, heads, v, vp, parts, ld_out, eps);
}
void launch_group_norm_rows(const SrcRows& y, const SrcRows& gate, int gcol, int mode, const float* w, void* out, bool f32,
                            int rows, int heads, int v, int vp, int parts, int ld_out, float eps, hipStream_t st) {
  if (f32) launch_group_norm<float>(y, gate, gcol, mode, w, out, rows, heads, v, vp, parts, ld_out, eps, st);
  else launch_group_norm<bf16_t>(y, gate, gcol, mode, w, out, rows, heads, v, vp, parts, ld_out, eps, st);
}

// Commit of one token per sequence, as commit_token_kernel does it, staging the scaled embedding row as
// the fp32 residual stream of the next step.  With logits: the first index of the row's maximum (NaN never
// wins), eight candidates per thread and pass in flight.
template <typename T>
__global__ __launch_bounds__(1024) void commit_rows_kernel(const float* __restrict__ logits, long long ld_logits,
                                                           int* __restrict__ sampled, const T* __restrict__ embed,
                                                           float scale, float* __restrict__ x, int* __restrict__ out_tokens,
                                                           int max_out, int* __restrict__ step, int* __restrict__ pos,
                                                           int* __restrict__ done, int* __restrict__ cur_token, int eos,
                                                           int ld, int vocab, const int* __restrict__ active) {
  __shared__ float sv[16];
  __shared__ int si[16];
  __shared__ int tok_s;
  const int b = blockIdx.x;
  if (active && !active[b]) return;
  if (logits) {
    const float* r = logits + b * ld_logits;
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    constexpr int U = 8;
    for (int i0 = threadIdx.x; i0 < vocab; i0 += 1024 * U) {
      float v[U];
#pragma unroll
      for (int u = 0; u < U; ++u) v[u] = r[min(i0 + u * 1024, vocab - 1)];
#pragma unroll
      for (int u = 0; u < U; ++u)
        if (i0 + u * 1024 < vocab && v[u] > bv) { bv = v[u]; bi = i0 + u * 1024; }    // a thread's indices ascend
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(bv, off, 64);
      const int oi = __shfl_xor(bi, off, 64);
      if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    if (lane == 0) { sv[wid] = bv; si[wid] = bi; }
    __syncthreads();
    if (threadIdx.x == 0) {
      for (int w = 1; w < 16; ++w)
        if (sv[w] > bv || (sv[w] == bv && si[w] < bi)) { bv = sv[w]; bi = si[w]; }
      tok_s = bi == 0x7fffffff ? 0 : bi;
      sampled[b] = tok_s;
    }
    __syncthreads();
  }
  int tok = logits ? tok_s : sampled[b];
  if (tok < 0 || tok >= vocab) tok = 0;
  for (int c = threadIdx.x * 8; c < ld; c += blockDim.x * 8) {
    float v[8];
    load8(embed + static_cast<long long>(tok) * ld + c, v);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= scale;
    store8(x + static_cast<long long>(b) * ld + c, v);
  }
  if (threadIdx.x == 0) {
    const int st = step[b];
    if (st >= 0 && st < max_out) out_tokens[static_cast<long long>(b) * max_out + st] = tok;
    cur_token[b] = tok;
    if (tok == eos) done[b] = 1;
    step[b] = st + 1;
    pos[b] = pos[b] + 1;
  }
}
void launch_commit_rows(const float* logits, long long ld_logits, int* sampled, const void* embed, bool f32, float scale,
                        float* x, int* out_tokens, int max_out, int* step, int* pos, int* done, int* cur_token, int eos, int B,
                        int ld, int vocab, const int* active, hipStream_t st) {
  const dim3 grid(B), block(logits ? 1024 : 256);
  if (f32)
    hipLaunchKernelGGL(commit_rows_kernel<float>, grid, block, 0, st, logits, ld_logits, sampled,
                       static_cast<const float*>(embed), scale, x, out_tokens, max_out, step, pos, done, cur_token, eos, ld,
                       vocab, active);
  else
    hipLaunchKernelGGL(commit_rows_kernel<bf16_t>, grid, block, 0, st, logits, ld_logits, sampled,
                       static_cast<const bf16_t*>(embed), scale, x, out_tokens, max_out, step, pos, done, cur_token, eos, ld,
                       vocab, active);
}

// Attention inputs of one row.  The q and k sections are read once, into LDS (STAGED; rows too wide for it are read
// again instead), where an element finds the one it is rotated with.
template <typename T, bool STAGED>
__global__ __launch_bounds__(256) void attn_prep_kernel(AttnPrepArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row_lds[];     // q section, k section
  __shared__ float red[16];
  const long long row = blockIdx.x;
  const int qn = a.Hq * a.D, kn = a.Hkv * a.D, half = a.rot >> 1;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * 8; c < qn; c += 2048) {
    float t[8];
    src8(a.src, row, a.q_col + c, t);
    sq += sumsq8(t);
    if constexpr (STAGED) store8(row_lds + c, t);
  }
  for (int c = threadIdx.x * 8; c < kn; c += 2048) {
    float t[8];
    src8(a.src, row, a.k_col + c, t);
    sk += sumsq8(t);
    if constexpr (STAGED) store8(row_lds + qn + c, t);
  }
  float v0[8];                                   // the first values are on their way while the sums meet
  if (threadIdx.x * 8 < static_cast<unsigned>(kn)) src8(a.src, row, a.v_col + threadIdx.x * 8, v0);
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) { red[threadIdx.x >> 6] = sq; red[8 + (threadIdx.x >> 6)] = sk; }
  __syncthreads();                               // (publishes the staged row too)
  const float rq = a.qw ? rsqrtf((red[0] + red[1] + red[2] + red[3]) / static_cast<float>(a.nq) + a.eps) : 1.f;
  const float rk = a.kw ? rsqrtf((red[8] + red[9] + red[10] + red[11]) / static_cast<float>(a.nk) + a.eps) : 1.f;
  const int p = a.row_pos[row];
  const int pt = min(max(p, 0), a.max_pos - 1);
  const float* cs = a.cos_tab + static_cast<long long>(pt) * half;
  const float* sn = a.sin_tab + static_cast<long long>(pt) * half;
  const long long slot = a.row_slot ? a.row_slot[row] : row;
  const bool keep = a.row_keep == nullptr || a.row_keep[row] != 0;
  const long long kv = a.row_kv ? a.row_kv[row] : -1;
  const int cslot = p % a.cap;
  // normalised and rotated elements c .. c + 7 (of one head) of a section
  auto value8 = [&](int col, int lds0, const float* w, float r, int c, float (&u)[8]) {
    const int d = c % a.D;
    auto raw1 = [&](int e) {
      const float v = STAGED ? row_lds[lds0 + e] : src1(a.src, row, col + e);
      return w ? v * r * w[e] : v * r;
    };
    auto raw8 = [&](int e, float (&v)[8]) {
      if constexpr (STAGED) load8(row_lds + lds0 + e, v);
      else src8(a.src, row, col + e, v);
      float g[8];
      if (w) load8(w + e, g);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] *= w ? r * g[i] : r;
    };
    raw8(c, u);
    if (d >= a.rot) return;
    if ((half & 7) == 0) {
      const bool lo = d < half;
      const int i0 = lo ? d : d - half;
      float o[8], cc[8], ss[8];
      raw8(lo ? c + half : c - half, o);
      load8(cs + i0, cc);
      load8(sn + i0, ss);
#pragma unroll
      for (int i = 0; i < 8; ++i) u[i] = lo ? u[i] * cc[i] - o[i] * ss[i] : u[i] * cc[i] + o[i] * ss[i];
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int e = d + i;
        if (e < half) u[i] = u[i] * cs[e] - raw1(c + i + half) * sn[e];
        else if (e < a.rot) u[i] = u[i] * cs[e - half] + raw1(c + i - half) * sn[e - half];
      }
    }
  };
  T* q = static_cast<T*>(a.q_out) + row * qn;
  for (int c = threadIdx.x * 8; c < qn; c += 2048) {
    float u[8];
    value8(a.q_col, 0, a.qw, rq, c, u);
    store8(q + c, u);
  }
  for (int c = threadIdx.x * 8; c < kn; c += 2048) {
    float u[8], v[8];
    value8(a.k_col, qn, a.kw, rk, c, u);
    if (c == static_cast<int>(threadIdx.x) * 8)
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = v0[i];
    else src8(a.src, row, a.v_col + c, v);
    if (kv >= 0) {
      store8(static_cast<T*>(a.k_buf) + kv * kn + c, u);
      store8(static_cast<T*>(a.v_buf) + kv * kn + c, v);
    }
    if (keep) {
      const long long o = ((slot * a.Hkv + c / a.D) * a.cap + cslot) * a.D + c % a.D;
      store8(static_cast<T*>(a.k_cache) + o, u);
      store8(static_cast<T*>(a.v_cache) + o, v);
    }
  }
}
void launch_attn_prep(const AttnPrepArgs& a, bool f32, int rows, hipStream_t st) {
  const size_t lds = static_cast<size_t>(a.Hq + a.Hkv) * a.D * 4;
  const bool staged = lds <= 64 * 1024;
  if (f32) {
    if (staged) hipLaunchKernelGGL((attn_prep_kernel<float, true>), dim3(rows), dim3(256), lds, st, a);
    else hipLaunchKernelGGL((attn_prep_kernel<float, false>), dim3(rows), dim3(256), 0, st, a);
  } else {
    if (staged) hipLaunchKernelGGL((attn_prep_kernel<bf16_t, true>), dim3(rows), dim3(256), lds, st, a);
    else hipLaunchKernelGGL((attn_prep_kernel<bf16_t, false>), dim3(rows), dim3(256), 0, st, a);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void chunk_keys_copy_kernel(const T* __restrict__ kc, const T* __restrict__ vc,
                                                              T* __restrict__ kb, T* __restrict__ vb,
                                                              const int* __restrict__ copies, int Hkv, int cap, int D) {
  const int* c = copies + blockIdx.y * 4;
  const long long slot = c[0];
  const int first = c[1], dst = c[2], count = c[3];
  for (int i = blockIdx.x; i < count; i += gridDim.x)
    for (int e = threadIdx.x; e < Hkv * D; e += 256) {
      const long long s = ((slot * Hkv + e / D) * cap + (first + i) % cap) * D + e % D;
      const long long o = static_cast<long long>(dst + i) * Hkv * D + e;
      kb[o] = kc[s];
      vb[o] = vc[s];
    }
}
void launch_chunk_keys_copy(const void* k_cache, const void* v_cache, void* k_buf, void* v_buf, const int* copies, int n,
                            bool f32, int Hkv, int cap, int D, hipStream_t st) {
  const dim3 grid(256, n);
  if (f32)
    hipLaunchKernelGGL(chunk_keys_copy_kernel<float>, grid, dim3(256), 0, st, static_cast<const float*>(k_cache),
                       static_cast<const float*>(v_cache), static_cast<float*>(k_buf), static_cast<float*>(v_buf), copies,
                       Hkv, cap, D);
  else
    hipLaunchKernelGGL(chunk_keys_copy_kernel<bf16_t>, grid, dim3(256), 0, st, static_cast<const bf16_t*>(k_cache),
                       static_cast<const bf16_t*>(v_cache), static_cast<bf16_t*>(k_buf), static_cast<bf16_t*>(v_buf),
                       copies, Hkv, cap, D);
}

// log gates of the matrix memory
__global__ __launch_bounds__(256) void mlstm_gates_kernel(SrcRows src, int i_col, int f_col,
                                                          const float* __restrict__ ib, const float* __restrict__ fb,
                                                          float cap, float* __restrict__ li, float* __restrict__ lf,
                                                          int total, int H) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int row = i / H, h = i % H;
  li[i] = cap * tanhf((src1(src, row, i_col + h) + ib[h]) / cap);
  const float f = cap * tanhf((src1(src, row, f_col + h) + fb[h]) / cap);
  lf[i] = -softplus_f(-f);
}
void launch_mlstm_gates(const SrcRows& src, int i_col, int f_col, const float* ib, const float* fb, float cap, float* li,
                        float* lf, int rows, int H, hipStream_t st) {
  const int total = rows * H;
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3((total + 255) / 256), dim3(256), 0, st, src, i_col, f_col, ib, fb, cap, li,
                     lf, total, H);
}

__global__ __launch_bounds__(256) void ssd_gates_kernel(SrcRows src, int col, const float* __restrict__ dt_bias,
                                                        const float* __restrict__ a_log, float* __restrict__ log_decay,
                                                        float* __restrict__ dt, int total, int H) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int row = i / H, h = i % H;
  const float d = softplus_f(src1(src, row, col + h) + dt_bias[h]);
  dt[i] = d;
  log_decay[i] = -expf(a_log[h]) * d;
}
void launch_ssd_gates(const SrcRows& src, int col, const float* dt_bias, const float* a_log, float* log_decay, float* dt,
                      int rows, int H, hipStream_t st) {
  const int total = rows * H;
  hipLaunchKernelGGL(ssd_gates_kernel, dim3((total + 255) / 256), dim3(256), 0, st, src, col, dt_bias, a_log, log_decay,
                     dt, total, H);
}

}  // namespace evgpt
