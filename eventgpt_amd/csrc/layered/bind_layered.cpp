// torch op registration for the layered decoders (namespace `evlay`), a library of its own (`_D.so`): a
// deployment of such a model builds these kernels and the shared GEMM / attention / sampling ones, nothing else.
// As in bind.cpp, operands are checked here so that no kernel is launched on shapes its indexing does not assume.
#include <algorithm>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <torch/library.h>

#include "../evgpt_kernels.h"
#include "../layered_kernels.h"

namespace {

using at::Tensor;
using OptTensor = c10::optional<Tensor>;
using evgpt::SrcRows;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

void check_t(const Tensor& t, const char* name) {       // storage type T: bf16 or fp32
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), name, " must be a contiguous GPU tensor");
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, name, " must be bfloat16 or float32");
  TORCH_CHECK((reinterpret_cast<uintptr_t>(t.data_ptr()) & 15) == 0, name, " must be 16-byte aligned");
}
bool is_f32(const Tensor& t) { return t.scalar_type() == at::kFloat; }
void check_f(const Tensor& t, const char* name) { check_t(t, name); TORCH_CHECK(is_f32(t), name, " must be float32"); }
void check_i(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt, name, " must be a contiguous int32 GPU tensor");
}
const float* fptr(const OptTensor& t) { return t.has_value() && t->defined() ? t->data_ptr<float>() : nullptr; }
const int* iptr(const OptTensor& t) { return t.has_value() && t->defined() ? t->data_ptr<int>() : nullptr; }
const evgpt::bf16_t* bptr(const Tensor& t) { return reinterpret_cast<const evgpt::bf16_t*>(t.data_ptr()); }
evgpt::bf16_t* bptr_mut(const Tensor& t) { return reinterpret_cast<evgpt::bf16_t*>(t.data_ptr()); }
at::ScalarType t_of(bool f32) { return f32 ? at::kFloat : at::kBFloat16; }

// rows of a projection: [M, ld] of either type (ld may be a row stride of a wider matrix), or fp32 slabs [S, M, ld]
SrcRows src_of(const Tensor& t, const char* name, int64_t* rows, int64_t* cols) {
  TORCH_CHECK(t.is_cuda() && (t.dim() == 2 || t.dim() == 3) && t.stride(-1) == 1, name, " must be [M, N] or [S, M, N]");
  TORCH_CHECK(t.scalar_type() == at::kFloat || (t.scalar_type() == at::kBFloat16 && t.dim() == 2), name, ": bf16 or fp32");
  const int64_t ld = t.stride(-2);
  TORCH_CHECK((reinterpret_cast<uintptr_t>(t.data_ptr()) & 15) == 0 && (t.size(-2) == 1 || ld % 8 == 0) && t.size(-1) % 8 == 0,
              name, ": rows must be aligned vectors of eight");
  *rows = t.size(-2);
  *cols = t.size(-1);
  return SrcRows{t.data_ptr(), t.dim() == 3 ? t.stride(0) : 0, t.dim() == 3 ? (int)t.size(0) : 1, (int)ld, is_f32(t)};
}

// ---------------------------------------------------------------- projections
Tensor linear(const Tensor& x, const Tensor& w, bool out_f32) {
  check_t(x, "x"); check_t(w, "w");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && x.scalar_type() == w.scalar_type(), "linear: x [M, K], w [N, K] of one type");
  const int64_t M = x.size(0), K = x.size(1), N = w.size(0);
  TORCH_CHECK(w.size(1) == K && K % 64 == 0 && K > 0 && N % 8 == 0, "linear: K % 64 == 0, N % 8 == 0");
  TORCH_CHECK(M * K < (1ll << 30) && N * K < (1ll << 30) && M * N < (1ll << 31), "linear: operands are addressed with 32-bit offsets");
  if (is_f32(x)) {
    Tensor y = at::empty({M, N}, x.options());
    if (M > 0)
      evgpt::launch_gemm_f32(x.data_ptr<float>(), w.data_ptr<float>(), y.data_ptr<float>(), (int)M, (int)N, (int)K, (int)K,
                             (int)K, (int)N, cur_stream());
    return y;
  }
  Tensor y = at::empty({M, N}, x.options().dtype(t_of(out_f32)));
  if (M == 0) return y;
  const int sk = evgpt::gemm_splitk((int)M, (int)N, (int)K);
  Tensor ws;
  if (sk > 1) {
    ws = at::empty({sk * M * N}, x.options().dtype(at::kFloat));
  } else {
    const int64_t tail = evgpt::gemm_tail_ws_floats((int)M, (int)N, (int)K);
    if (tail > 0) ws = at::empty({tail}, x.options().dtype(at::kFloat));
  }
  evgpt::launch_gemm_bf16(bptr(x), bptr(w), out_f32 ? nullptr : bptr_mut(y), out_f32 ? y.data_ptr<float>() : nullptr, nullptr,
                          nullptr, (int)M, (int)N, (int)K, (int)K, (int)K, (int)N, 0, nullptr, nullptr,
                          ws.defined() ? ws.data_ptr<float>() : nullptr, sk, cur_stream());
  return y;
}

// fp32 split-K slabs [S, M, N] for a consumer that sums them (fp32 operands: one slab)
Tensor linear_slabs(const Tensor& x, const Tensor& w) {
  if (is_f32(x)) return linear(x, w, true).unsqueeze(0);
  check_t(x, "x"); check_t(w, "w");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && !is_f32(w), "linear_slabs: x [M, K], w [N, K] of one type");
  const int64_t M = x.size(0), K = x.size(1), N = w.size(0);
  TORCH_CHECK(M >= 1 && w.size(1) == K && K % 64 == 0 && K > 0 && N % 8 == 0, "linear_slabs: K % 64 == 0, N % 8 == 0");
  TORCH_CHECK(M * K < (1ll << 30) && N * K < (1ll << 30), "linear_slabs: operands are addressed with 32-bit offsets");
  const int sk = evgpt::gemm_splitk_slabs((int)M, (int)N, (int)K);
  Tensor ws = at::empty({sk, M, N}, x.options().dtype(at::kFloat));
  const int used = evgpt::launch_gemm_partial(bptr(x), bptr(w), ws.data_ptr<float>(), (int)M, (int)N, (int)K, (int)K, (int)K,
                                              cur_stream(), 0);
  return used == sk ? ws : ws.narrow(0, 0, used);
}

// act(x Wgate^T) * (x Wup^T), w_gate_up [2 I, K]; bf16: the activation in the GEMM's epilogue
Tensor linear_glu(const Tensor& x, const Tensor& w, int64_t act) {
  TORCH_CHECK(act == evgpt::GLU_GELU_TANH || act == evgpt::GLU_SILU, "linear_glu: act 0 or 1");
  TORCH_CHECK(w.dim() == 2 && w.size(0) % 64 == 0, "linear_glu: w_gate_up [2 I, K], I % 32 == 0");
  const int64_t I = w.size(0) / 2;
  if (is_f32(x) || x.size(0) <= 32) {
    const Tensor y = is_f32(x) ? linear(x, w, true) : linear_slabs(x, w);
    Tensor h = at::empty({x.size(0), I}, x.options());
    const SrcRows s{y.data_ptr(), y.dim() == 3 ? y.stride(0) : 0, y.dim() == 3 ? (int)y.size(0) : 1, (int)(2 * I), 1};
    evgpt::launch_glu_rows(s, h.data_ptr(), is_f32(x), (int)x.size(0), (int)I, (int)act, cur_stream());
    return h;
  }
  check_t(x, "x"); check_t(w, "w");
  const int64_t M = x.size(0), K = x.size(1);
  TORCH_CHECK(x.dim() == 2 && !is_f32(w) && w.size(1) == K && K % 64 == 0 && K > 0, "linear_glu: x [M, K], K % 64 == 0");
  TORCH_CHECK(2 * I * K * 2 < (1ll << 31) && M * K * 2 < (1ll << 31), "linear_glu: operands over 2 GiB");
  Tensor h = at::empty({M, I}, x.options());
  evgpt::launch_gemm_glu(bptr(x), bptr(w), bptr_mut(h), (int)M, (int)I, (int)K, (int)K, (int)K, (int)I, cur_stream(),
                         act == evgpt::GLU_SILU ? 0 : 1);
  return h;
}

// ---------------------------------------------------------------- rows
Tensor embed_rows(const Tensor& tok, const Tensor& embed, double scale) {
  check_i(tok, "tokens"); check_t(embed, "embed");
  TORCH_CHECK(embed.dim() == 2 && embed.size(1) % 64 == 0, "embed: [V, padded width]");
  const int64_t M = tok.numel(), ld = embed.size(1);
  Tensor x = at::empty({M, ld}, embed.options().dtype(at::kFloat));
  if (M > 0)
    evgpt::launch_embed_rows(tok.data_ptr<int>(), embed.data_ptr(), is_f32(embed), (float)scale, x.data_ptr<float>(), (int)M,
                             (int)ld, (int)embed.size(0), cur_stream());
  return x;
}

void check_stream(const Tensor& x, int64_t n) {
  check_f(x, "x");
  TORCH_CHECK(x.dim() == 2 && x.size(1) % 64 == 0 && n >= 1 && n <= x.size(1), "x: [M, padded width]");
}
Tensor norm_rows(const Tensor& x, const OptTensor& sel, const Tensor& w, int64_t n, double eps, bool f32, bool layer) {
  check_stream(x, n); check_f(w, "w");
  TORCH_CHECK(w.numel() == x.size(1), "norm_rows: weight size");
  if (sel.has_value()) check_i(*sel, "sel");
  const int64_t M = sel.has_value() ? sel->numel() : x.size(0);
  Tensor xn = at::empty({M, x.size(1)}, x.options().dtype(t_of(f32)));
  if (M > 0)
    evgpt::launch_norm_rows(x.data_ptr<float>(), iptr(sel), w.data_ptr<float>(), xn.data_ptr(), f32, (int)M, (int)n,
                            (int)x.size(1), (float)eps, layer, cur_stream());
  return xn;
}
SrcRows stream_src(const Tensor& y, const Tensor& x, const char* name) {
  int64_t r, c;
  const SrcRows s = src_of(y, name, &r, &c);
  TORCH_CHECK(r == x.size(0) && c >= x.size(1), name, ": rows of the residual stream");
  return s;
}
Tensor xn_of(const Tensor& x, const OptTensor& w, bool f32) {
  if (!w.has_value()) return at::empty({0}, x.options().dtype(t_of(f32)));
  check_f(*w, "w");
  TORCH_CHECK(w->numel() == x.size(1), "norm weight size");
  return at::empty({x.size(0), x.size(1)}, x.options().dtype(t_of(f32)));
}
Tensor add_norm_rows_(const Tensor& x, const Tensor& y, const OptTensor& w, int64_t n, double eps, bool f32, bool layer) {
  check_stream(x, n);
  const SrcRows s = stream_src(y, x, "y");
  Tensor xn = xn_of(x, w, f32);
  evgpt::launch_add_norm_rows(x.data_ptr<float>(), s, fptr(w), xn.data_ptr(), f32, (int)x.size(0), (int)n, (int)x.size(1),
                              (float)eps, layer, cur_stream());
  return xn;
}
// x += norm(y) * wy; norm of the new x * w
Tensor post_norm_rows_(const Tensor& x, const Tensor& y, const Tensor& wy, const OptTensor& w, int64_t n, double eps, bool f32,
                       bool layer) {
  check_stream(x, n); check_f(wy, "wy");
  TORCH_CHECK(wy.numel() == x.size(1), "post_norm_rows: weight size");
  const SrcRows s = stream_src(y, x, "y");
  Tensor xn = xn_of(x, w, f32);
  if (x.size(0) > 0)
    evgpt::launch_post_norm_rows(x.data_ptr<float>(), s, wy.data_ptr<float>(), fptr(w), xn.data_ptr(), f32, (int)x.size(0), (int)n,
                                 (int)x.size(1), (float)eps, layer, cur_stream());
  return xn;
}
// the same with y[row] = sum_k weights[row][k] * y[pick[row][k]] (without wy: x += y)
Tensor mix_norm_rows_(const Tensor& x, const Tensor& y, const Tensor& pick, const Tensor& weights, const OptTensor& wy,
                      const OptTensor& w, int64_t n, double eps, bool f32, bool layer) {
  check_stream(x, n); check_t(y, "y"); check_i(pick, "pick"); check_f(weights, "weights");
  TORCH_CHECK(y.dim() == 2 && y.size(1) >= x.size(1) && y.size(1) % 8 == 0 && is_f32(y) == f32, "mix_norm_rows: y [rows, width]");
  TORCH_CHECK(weights.dim() == 2 && weights.size(0) == x.size(0) && weights.size(1) >= 1 && pick.numel() == weights.numel(),
              "mix_norm_rows: pick, weights [M, top]");
  if (wy.has_value()) { check_f(*wy, "wy"); TORCH_CHECK(wy->numel() == x.size(1), "mix_norm_rows: weight size"); }
  Tensor xn = xn_of(x, w, f32);
  const evgpt::MixRows m{y.data_ptr(), pick.data_ptr<int>(), weights.data_ptr<float>(), (int)weights.size(1), (int)y.size(1)};
  if (x.size(0) > 0)
    evgpt::launch_mix_norm_rows(x.data_ptr<float>(), m, fptr(wy), fptr(w), xn.data_ptr(), f32, (int)x.size(0), (int)n,
                                (int)x.size(1), (float)eps, layer, cur_stream());
  return xn;
}
void cap_logits_(const Tensor& x, double scale, double cap) {
  check_f(x, "logits");
  TORCH_CHECK(x.numel() % 4 == 0 && cap >= 0, "cap_logits: a multiple of four values, cap >= 0");
  if (x.numel() > 0) evgpt::launch_cap_logits(x.data_ptr<float>(), x.numel(), (float)scale, (float)cap, cur_stream());
}
Tensor merge_norm_rows_(const Tensor& x, const Tensor& a, const Tensor& b, const Tensor& wa, const Tensor& wb,
                        const OptTensor& w, int64_t n, double eps, bool f32) {
  check_stream(x, n); check_f(wa, "wa"); check_f(wb, "wb");
  TORCH_CHECK(wa.numel() == x.size(1) && wb.numel() == x.size(1), "merge_norm_rows: branch weights");
  const SrcRows sa = stream_src(a, x, "a"), sb = stream_src(b, x, "b");
  Tensor xn = xn_of(x, w, f32);
  evgpt::launch_merge_norm_rows(x.data_ptr<float>(), sa, sb, wa.data_ptr<float>(), wb.data_ptr<float>(), fptr(w),
                                xn.data_ptr(), f32, (int)x.size(0), (int)n, (int)x.size(1), (float)eps, cur_stream());
  return xn;
}
Tensor glu_rows(const Tensor& src, int64_t act, bool f32) {
  int64_t M, N;
  const SrcRows s = src_of(src, "src", &M, &N);
  TORCH_CHECK(N % 16 == 0 && (act == evgpt::GLU_GELU_TANH || act == evgpt::GLU_SILU), "glu_rows: [M, 2 I], act 0 or 1");
  Tensor h = at::empty({M, N / 2}, src.options().dtype(t_of(f32)));
  evgpt::launch_glu_rows(s, h.data_ptr(), f32, (int)M, (int)(N / 2), (int)act, cur_stream());
  return h;
}
// y: [M, heads * vp] rows of either type; gate_mode 0 none, 1 silu before the norm, 2 sigmoid after it
Tensor group_norm_rows(const Tensor& y, const OptTensor& gate, int64_t gcol, int64_t gate_mode, const Tensor& w, int64_t heads,
                       int64_t v, int64_t vp, int64_t parts, int64_t ld_out, double eps, bool f32) {
  check_f(w, "w");
  int64_t M, N, gm, gn;
  const SrcRows ys = src_of(y, "y", &M, &N);
  TORCH_CHECK(N == heads * vp && w.numel() == heads * vp && vp % 8 == 0 && v >= 1 && v <= vp, "group_norm_rows: y [M, heads * vp]");
  SrcRows gs{};
  TORCH_CHECK(gate_mode >= 0 && gate_mode <= 2 && (gate_mode == 0 || gate.has_value()), "group_norm_rows: gate");
  if (gate_mode) {
    gs = src_of(*gate, "gate", &gm, &gn);
    TORCH_CHECK(gm == M && gcol >= 0 && gcol % 8 == 0 && gcol + heads * vp <= gn, "group_norm_rows: gate columns");
  }
  TORCH_CHECK(parts >= 1 && heads * v % parts == 0 && ld_out % 8 == 0 && ld_out >= heads * vp, "group_norm_rows: parts, ld_out");
  TORCH_CHECK((heads * vp + parts) * 4 <= 150 * 1024, "group_norm_rows: row too wide for LDS");
  Tensor o = at::empty({M, ld_out}, w.options().dtype(t_of(f32)));
  if (M > 0)
    evgpt::launch_group_norm_rows(ys, gs, (int)gcol, (int)gate_mode, w.data_ptr<float>(), o.data_ptr(), f32, (int)M, (int)heads,
                                  (int)v, (int)vp, (int)parts, (int)ld_out, (float)eps, cur_stream());
  return o;
}
// logits [B, >= V] fp32: greedy, `sampled` receives the tokens; without: `sampled` holds them
void commit_rows_(const OptTensor& logits, const Tensor& sampled, const Tensor& embed, double scale, const Tensor& x, const Tensor& out_tokens,
                  const Tensor& step, const Tensor& pos, const Tensor& done, const Tensor& cur, int64_t eos,
                  const OptTensor& active) {
  check_i(sampled, "sampled"); check_t(embed, "embed"); check_f(x, "x"); check_i(out_tokens, "out_tokens");
  check_i(step, "step"); check_i(pos, "pos"); check_i(done, "done"); check_i(cur, "cur_token");
  const int64_t B = x.size(0);
  TORCH_CHECK(embed.dim() == 2 && embed.size(1) == x.size(1) && x.size(1) % 64 == 0, "commit_rows: embedding width");
  TORCH_CHECK(sampled.numel() >= B && step.numel() >= B && pos.numel() >= B && done.numel() >= B && cur.numel() >= B &&
              out_tokens.dim() == 2 && out_tokens.size(0) >= B, "commit_rows: per-sequence buffers");
  if (active.has_value()) { check_i(*active, "active"); TORCH_CHECK(active->numel() >= B, "active"); }
  if (logits.has_value())
    TORCH_CHECK(logits->is_cuda() && logits->dim() == 2 && is_f32(*logits) && logits->stride(1) == 1 && logits->size(0) == B &&
                logits->size(1) >= embed.size(0), "commit_rows: logits [B, V] fp32");
  evgpt::launch_commit_rows(fptr(logits), logits.has_value() ? logits->stride(0) : 0, sampled.data_ptr<int>(), embed.data_ptr(), is_f32(embed), (float)scale, x.data_ptr<float>(),
                            out_tokens.data_ptr<int>(), (int)out_tokens.size(1), step.data_ptr<int>(), pos.data_ptr<int>(),
                            done.data_ptr<int>(), cur.data_ptr<int>(), (int)eos, (int)B, (int)x.size(1),
                            (int)embed.size(0), iptr(active), cur_stream());
}
void sample_top_p(const Tensor& logits, const Tensor& out, double temperature, double top_p, int64_t seed,
                  const Tensor& step, int64_t top_k) {
  check_f(logits, "logits"); check_i(out, "out"); check_i(step, "step");
  TORCH_CHECK(logits.dim() == 2 && out.numel() >= logits.size(0) && step.numel() >= logits.size(0) && temperature > 0,
              "sample_top_p: logits [B, V], temperature > 0");
  evgpt::launch_sample_top_p(logits.data_ptr<float>(), out.data_ptr<int>(), (int)logits.size(0), (int)logits.size(1),
                             (float)temperature, (int)top_k, (float)top_p, (unsigned long long)seed, step.data_ptr<int>(),
                             cur_stream());
}

// ---------------------------------------------------------------- attention
// the heads of an attention layer: columns of its sections in a projection, norms, rotation tables, chunk cache
evgpt::AttnPrepArgs prep_args(const SrcRows& src, int64_t M, int64_t N, int64_t q_col, int64_t k_col, int64_t v_col,
                              const OptTensor& qw, const OptTensor& kw, int64_t Hq, int64_t Hkv, int64_t D, int64_t nq, int64_t nk,
                              double eps, const Tensor& cos, const Tensor& sin, const Tensor& row_pos, const Tensor& k_cache,
                              const Tensor& v_cache) {
  evgpt::AttnPrepArgs a{};
  a.src = src;
  check_t(k_cache, "k_cache"); check_t(v_cache, "v_cache");
  TORCH_CHECK(Hq >= 1 && Hkv >= 1 && Hq % Hkv == 0 && D % 64 == 0 && D >= 64, "attention: heads");
  TORCH_CHECK(q_col % 8 == 0 && k_col % 8 == 0 && v_col % 8 == 0 && q_col >= 0 && k_col >= 0 && v_col >= 0 &&
              q_col + Hq * D <= N && k_col + Hkv * D <= N && v_col + Hkv * D <= N, "attention: sections");
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.sizes() == v_cache.sizes() && k_cache.size(1) == Hkv && k_cache.size(3) == D &&
              k_cache.size(2) >= 1 && v_cache.scalar_type() == k_cache.scalar_type(), "attention: caches [slots, Hkv, cap, D]");
  check_f(cos, "cos"); check_f(sin, "sin");
  TORCH_CHECK(cos.dim() == 2 && cos.sizes() == sin.sizes() && cos.size(0) >= 1 && cos.size(1) * 2 <= D, "attention: rotation tables");
  check_i(row_pos, "row_pos");
  TORCH_CHECK(row_pos.numel() >= M, "attention: row_pos");
  if (qw.has_value()) { check_f(*qw, "qw"); TORCH_CHECK(qw->numel() == Hq * D && nq >= 1); }
  if (kw.has_value()) { check_f(*kw, "kw"); TORCH_CHECK(kw->numel() == Hkv * D && nk >= 1); }
  a.q_col = (int)q_col; a.k_col = (int)k_col; a.v_col = (int)v_col;
  a.qw = fptr(qw); a.kw = fptr(kw);
  a.Hq = (int)Hq; a.Hkv = (int)Hkv; a.D = (int)D; a.nq = (int)nq; a.nk = (int)nk; a.eps = (float)eps;
  a.cos_tab = cos.data_ptr<float>(); a.sin_tab = sin.data_ptr<float>();
  a.rot = (int)cos.size(1) * 2; a.max_pos = (int)cos.size(0);
  a.row_pos = row_pos.data_ptr<int>();
  a.k_cache = k_cache.data_ptr(); a.v_cache = v_cache.data_ptr(); a.cap = (int)k_cache.size(2);
  return a;
}

// returns q [M, Hq, D]; k_buf / v_buf and / or the chunk cache are written in place
Tensor attn_prep_(const Tensor& src, int64_t q_col, int64_t k_col, int64_t v_col, const OptTensor& qw, const OptTensor& kw,
                  int64_t Hq, int64_t Hkv, int64_t D, int64_t nq, int64_t nk, double eps, const Tensor& cos, const Tensor& sin,
                  const OptTensor& row_slot, const Tensor& row_pos, const OptTensor& row_kv, const OptTensor& row_keep,
                  const OptTensor& k_buf, const OptTensor& v_buf, const Tensor& k_cache, const Tensor& v_cache) {
  int64_t M, N;
  const SrcRows rows = src_of(src, "src", &M, &N);
  evgpt::AttnPrepArgs a = prep_args(rows, M, N, q_col, k_col, v_col, qw, kw, Hq, Hkv, D, nq, nk, eps, cos, sin, row_pos,
                                    k_cache, v_cache);
  const bool f32 = is_f32(k_cache);
  if (row_slot.has_value()) { check_i(*row_slot, "row_slot"); TORCH_CHECK(row_slot->numel() == M); }
  else TORCH_CHECK(M <= k_cache.size(0), "attn_prep: more rows than cache slots");
  if (row_keep.has_value()) { check_i(*row_keep, "row_keep"); TORCH_CHECK(row_keep->numel() == M); }
  if (row_kv.has_value()) {
    check_i(*row_kv, "row_kv");
    TORCH_CHECK(row_kv->numel() == M && k_buf.has_value() && v_buf.has_value(), "attn_prep: key buffer");
    check_t(*k_buf, "k_buf"); check_t(*v_buf, "v_buf");
    TORCH_CHECK(k_buf->numel() % (Hkv * D) == 0 && k_buf->numel() >= M * Hkv * D && v_buf->numel() == k_buf->numel() &&
                is_f32(*k_buf) == f32 && is_f32(*v_buf) == f32, "attn_prep: key buffer size");
    a.k_buf = k_buf->data_ptr();
    a.v_buf = v_buf->data_ptr();
  }
  Tensor q = at::empty({M, Hq, D}, k_cache.options());
  a.row_slot = iptr(row_slot); a.row_kv = iptr(row_kv); a.row_keep = iptr(row_keep);
  a.q_out = q.data_ptr();
  if (M > 0) evgpt::launch_attn_prep(a, f32, (int)M, cur_stream());
  return q;
}
void chunk_keys_copy_(const Tensor& k_cache, const Tensor& v_cache, const Tensor& k_buf, const Tensor& v_buf, const Tensor& copies) {
  check_t(k_cache, "k_cache"); check_t(v_cache, "v_cache"); check_t(k_buf, "k_buf"); check_t(v_buf, "v_buf"); check_i(copies, "copies");
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.sizes() == v_cache.sizes() && copies.dim() == 2 && copies.size(1) == 4 &&
              copies.size(0) < 65536, "chunk_keys_copy: copies [n, 4]");
  TORCH_CHECK(is_f32(k_cache) == is_f32(k_buf) && is_f32(v_cache) == is_f32(v_buf) && is_f32(k_buf) == is_f32(v_buf), "chunk_keys_copy: types");
  if (copies.size(0) > 0)
    evgpt::launch_chunk_keys_copy(k_cache.data_ptr(), v_cache.data_ptr(), k_buf.data_ptr(), v_buf.data_ptr(),
                                  copies.data_ptr<int>(), (int)copies.size(0), is_f32(k_cache), (int)k_cache.size(1),
                                  (int)k_cache.size(2), (int)k_cache.size(3), cur_stream());
}
// k, v: rows of [Hkv][D]; the rows may be strided (columns of a wider matrix)
void check_qkv(const Tensor& q, const Tensor& k, const Tensor& v) {
  check_t(q, "q");
  TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && k.sizes() == v.sizes() && q.size(2) == k.size(2) && q.size(1) % k.size(1) == 0 &&
              q.scalar_type() == k.scalar_type() && q.scalar_type() == v.scalar_type(), "attention: q [M, Hq, D], k / v [R, Hkv, D]");
  TORCH_CHECK(q.size(2) % 64 == 0 && q.size(2) <= 512, "attention: head size a multiple of 64 up to 512");
  for (const Tensor* t : {&k, &v})
    TORCH_CHECK(t->is_cuda() && t->stride(2) == 1 && (t->size(1) == 1 || t->stride(1) == t->size(2)) && t->stride(0) % 8 == 0 &&
                t->stride(0) >= t->size(1) * t->size(2) && t->stride(0) == k.stride(0) &&
                (reinterpret_cast<uintptr_t>(t->data_ptr()) & 15) == 0, "attention: k, v: aligned rows of heads");
}
// rows of a matrix of q's type whose columns gcol .. gcol + Hq gate the heads
const void* head_gates(const OptTensor& gate, int64_t gcol, const Tensor& q, int64_t* ld) {
  *ld = 0;
  if (!gate.has_value()) return nullptr;
  TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 && gate->stride(1) == 1 && gate->scalar_type() == q.scalar_type() &&
              gate->size(0) == q.size(0) && gcol >= 0 && gcol + q.size(1) <= gate->size(1), "attention: gate [M, N]");
  *ld = gate->stride(0);
  return static_cast<const char*>(gate->data_ptr()) + gcol * (is_f32(q) ? 4 : 2);
}
Tensor attn_chunk(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& items, double scale, const OptTensor& gate,
                  int64_t gcol) {
  check_qkv(q, k, v); check_i(items, "items");
  TORCH_CHECK(items.dim() == 2 && items.size(1) == 4, "attn_chunk: items [n, 4]");
  int64_t gld;
  const void* g = head_gates(gate, gcol, q, &gld);
  Tensor o = at::empty_like(q);
  if (items.size(0) > 0)
    evgpt::launch_attn_chunk(q.data_ptr(), k.data_ptr(), v.data_ptr(), o.data_ptr(), items.data_ptr<int>(), (int)items.size(0),
                             is_f32(q), (int)q.size(1), (int)k.size(1), (int)q.size(2), k.stride(0), (float)scale, g, (int)gld,
                             cur_stream());
  return o;
}
// `n` equal runs of `rows` query rows starting at q0, each with its keys `stride` key rows after the one before, the
// run's first query at position `off` of its chunk, on the flash kernel (bf16, head size 64 or 128)
void attn_runs_(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& o, int64_t q0, int64_t rows, int64_t kv0,
                int64_t off, int64_t n, double scale, const OptTensor& gate, int64_t gcol) {
  check_qkv(q, k, v); check_t(o, "o");
  const int64_t Hq = q.size(1), Hkv = k.size(1), D = q.size(2);
  TORCH_CHECK(!is_f32(q) && (D == 64 || D == 128) && o.sizes() == q.sizes() && !is_f32(o), "attn_runs: bf16, head size 64 or 128");
  TORCH_CHECK(rows >= 1 && n >= 1 && q0 >= 0 && kv0 >= 0 && off >= 0 && (n == 1 || off == 0) && q0 + n * rows <= q.size(0) &&
              kv0 + off + n * rows <= k.size(0), "attn_runs: rows");
  const long long ks = k.stride(0);
  int64_t gld;
  const evgpt::bf16_t* g = static_cast<const evgpt::bf16_t*>(head_gates(gate, gcol, q, &gld));
  const long long st[12] = {rows * Hq * D, Hq * D, D, rows * ks, ks, D, rows * ks, ks, D, rows * Hq * D, Hq * D, D};
  evgpt::launch_attn_prefill(bptr(q) + q0 * Hq * D, bptr(k) + kv0 * ks, bptr(v) + kv0 * ks, bptr_mut(o) + q0 * Hq * D,
                             st, nullptr, (int)n, (int)rows, (int)(off + rows), (int)Hq, (int)Hkv, (int)D, 1, (int)off, 0,
                             (float)scale, cur_stream(), nullptr, nullptr, 0, nullptr, true, g ? g + q0 * gld : nullptr, (int)gld);
}
// split-KV decode attention of the other models on the chunk cache (bf16, head size 64 or 128); part_o / part_ml: scratch
Tensor attn_chunk_decode(const Tensor& q, const Tensor& k_cache, const Tensor& v_cache, const Tensor& pos, double scale,
                         int64_t nsplit) {
  check_t(q, "q"); check_t(k_cache, "k_cache"); check_t(v_cache, "v_cache"); check_i(pos, "pos");
  TORCH_CHECK(q.dim() == 3 && k_cache.dim() == 4 && k_cache.sizes() == v_cache.sizes(), "attn_chunk_decode: shapes");
  const int64_t B = q.size(0), Hq = q.size(1), D = q.size(2), Hkv = k_cache.size(1), cap = k_cache.size(2);
  TORCH_CHECK(k_cache.size(0) >= B && k_cache.size(3) == D && Hq % Hkv == 0 && pos.numel() >= B && D % 64 == 0 && D <= 512 &&
              q.scalar_type() == k_cache.scalar_type() && q.scalar_type() == v_cache.scalar_type(), "attn_chunk_decode: shapes");
  Tensor o = at::empty_like(q);
  if (!is_f32(q) && (D == 64 || D == 128)) {
    nsplit = std::min<int64_t>(std::max<int64_t>(nsplit, 1), 16);
    auto f = q.options().dtype(at::kFloat);
    Tensor po = at::empty({nsplit > 1 ? B * Hq * nsplit * D : 1}, f), pm = at::empty({nsplit > 1 ? B * Hq * nsplit * 2 : 1}, f);
    evgpt::launch_attn_decode(bptr(q), bptr(k_cache), bptr(v_cache), bptr_mut(o), po.data_ptr<float>(), pm.data_ptr<float>(),
                              pos.data_ptr<int>(), (int)B, (int)Hq, (int)Hkv, (int)D, (int)cap, (int)nsplit, (float)scale,
                              cur_stream(), 1);
    return o;
  }
  evgpt::launch_attn_chunk_decode(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), o.data_ptr(), nullptr, pos.data_ptr<int>(),
                                  is_f32(q), (int)B, (int)Hq, (int)Hkv, (int)D, (int)cap, (float)scale, cur_stream());
  return o;
}

// ---------------------------------------------------------------- recurrences
// q / k / v: 2-D views (rows, columns from the head section's start) of T matrices
evgpt::ScanArgs scan_args(const Tensor& q, const Tensor& k, const Tensor& v, int64_t H, int64_t per_group, int64_t N, int64_t V,
                          double qscale, const Tensor& log_decay, const OptTensor& log_in, const OptTensor& scale_in,
                          const OptTensor& skip, const Tensor& S, const OptTensor& n, const OptTensor& m) {
  const int64_t M = q.size(0);
  auto view = [&](const Tensor& t, int64_t cols, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.stride(1) == 1 && t.size(0) == M && t.size(1) >= cols && t.scalar_type() == q.scalar_type() &&
                (M <= 1 || t.stride(0) % 8 == 0) && (reinterpret_cast<uintptr_t>(t.data_ptr()) & 15) == 0, name, ": aligned rows of one type");
  };
  TORCH_CHECK(q.scalar_type() == at::kBFloat16 || q.scalar_type() == at::kFloat, "scan: bf16 or fp32");
  TORCH_CHECK(H >= 1 && per_group >= 1 && H % per_group == 0 && N >= 32 && N % 32 == 0 && (V == 32 || (V >= 64 && V % 64 == 0)), "scan: sizes");
  view(q, H / per_group * N, "q"); view(k, H / per_group * N, "k"); view(v, H * V, "v");
  check_f(log_decay, "log_decay");
  TORCH_CHECK(log_decay.numel() == M * H, "scan: log_decay [M, H]");
  TORCH_CHECK(log_in.has_value() != scale_in.has_value(), "scan: log_in or scale_in");
  if (log_in.has_value()) {
    check_f(*log_in, "log_in");
    TORCH_CHECK(log_in->numel() == M * H && n.has_value() && m.has_value(), "scan: log_in [M, H], normaliser, maximum");
    check_f(*n, "n"); check_f(*m, "m");
    TORCH_CHECK(n->numel() == 2 * S.size(0) * H * N && m->numel() == 2 * S.size(0) * H, "scan: normaliser, maximum [2, slots, ..]");
  } else {
    check_f(*scale_in, "scale_in");
    TORCH_CHECK(scale_in->numel() == M * H, "scan: scale_in [M, H]");
  }
  if (skip.has_value()) { check_f(*skip, "skip"); TORCH_CHECK(skip->numel() == H, "scan: skip [H]"); }
  check_f(S, "S");
  TORCH_CHECK(S.dim() == 4 && S.size(1) == H && S.size(2) == V && S.size(3) == N, "scan: S [slots, H, V, N]");
  evgpt::ScanArgs a{};
  a.q = q.data_ptr(); a.k = k.data_ptr(); a.v = v.data_ptr();
  a.ldq = q.stride(0); a.ldk = k.stride(0); a.ldv = v.stride(0);
  a.per_group = (int)per_group; a.H = (int)H; a.N = (int)N; a.V = (int)V; a.qscale = (float)qscale;
  a.log_decay = log_decay.data_ptr<float>(); a.log_in = fptr(log_in); a.scale_in = fptr(scale_in); a.skip = fptr(skip);
  a.S = S.data_ptr<float>();
  a.n = const_cast<float*>(fptr(n)); a.m = const_cast<float*>(fptr(m));
  a.slots = (int)S.size(0);
  return a;
}
Tensor scan_prefill_(const Tensor& q, const Tensor& k, const Tensor& v, int64_t H, int64_t per_group, int64_t N, int64_t V,
                     double qscale, const Tensor& log_decay, const OptTensor& log_in, const OptTensor& scale_in, const OptTensor& skip,
                     const Tensor& S, const OptTensor& n, const OptTensor& m, const Tensor& chunks, const Tensor& seqs) {
  evgpt::ScanArgs a = scan_args(q, k, v, H, per_group, N, V, qscale, log_decay, log_in, scale_in, skip, S, n, m);
  check_i(chunks, "chunks"); check_i(seqs, "seqs");
  TORCH_CHECK(chunks.dim() == 2 && chunks.size(1) == 4 && seqs.dim() == 2 && seqs.size(1) == 4, "scan: tables [n, 4]");
  const int64_t C = chunks.size(0);
  TORCH_CHECK(C < 65536 && H < 65536 && seqs.size(0) < 65536, "scan: grid");
  Tensor o = at::empty({q.size(0), H * V}, q.options());
  if (C == 0) return o;
  auto f = q.options().dtype(at::kFloat);
  Tensor dS = at::empty({C, H, V, N}, f), dn = at::empty({C, H, N}, f), m0 = at::empty({C, H}, f);
  Tensor sc = at::empty({2, C, H}, f.dtype(at::kDouble));
  evgpt::ScanChunks c{chunks.data_ptr<int>(), seqs.data_ptr<int>(), (int)C, (int)seqs.size(0), dS.data_ptr<float>(),
                      dn.data_ptr<float>(), sc.data_ptr<double>(), sc.data_ptr<double>() + C * H, m0.data_ptr<float>()};
  a.out = o.data_ptr();
  evgpt::launch_scan_prefill(a, c, is_f32(q), cur_stream());
  return o;
}
// ---------------------------------------------------------------- decode steps
// One token per sequence from the projection rows `src`: the attention heads (norm, rotation, cache append; q is
// returned) and the matrix memory (its output is returned, fp32).  Rows whose `live` is 0 change no state.
std::tuple<Tensor, Tensor> parallel_step_(const Tensor& src, at::IntArrayRef attn, const OptTensor& qw, const OptTensor& kw,
                                          double eps, const Tensor& cos, const Tensor& sin, const Tensor& k_cache, const Tensor& v_cache,
                                          at::IntArrayRef mem, const Tensor& ib, const Tensor& fb, double cap, double qscale,
                                          const Tensor& S, const Tensor& n, const Tensor& m, const Tensor& pos, const OptTensor& live) {
  int64_t B, N;
  const SrcRows rows = src_of(src, "src", &B, &N);
  TORCH_CHECK(attn.size() == 8 && mem.size() == 8, "parallel_step: attn {q, k, v columns, Hq, Hkv, D, true q, true k widths}, "
              "mem {q, k, v, i, f columns, H, N, V}");
  evgpt::StepHeads sh{};
  sh.a = prep_args(rows, B, N, attn[0], attn[1], attn[2], qw, kw, attn[3], attn[4], attn[5], attn[6], attn[7], eps, cos, sin, pos,
                   k_cache, v_cache);
  sh.on = 1;
  const bool f32 = is_f32(k_cache);
  const int64_t H = mem[5], Nq = mem[6], V = mem[7];
  check_f(ib, "ib"); check_f(fb, "fb"); check_f(S, "S"); check_f(n, "n"); check_f(m, "m");
  TORCH_CHECK(H >= 1 && Nq >= 32 && Nq % 32 == 0 && Nq <= 4096 && (V == 32 || (V >= 64 && V % 64 == 0)) && cap > 0, "parallel_step: memory sizes");
  for (int i = 0; i < 3; ++i)
    TORCH_CHECK(mem[i] >= 0 && mem[i] + H * (i == 2 ? V : Nq) <= N, "parallel_step: memory sections");
  TORCH_CHECK(mem[3] >= 0 && mem[4] >= 0 && mem[3] + H <= N && mem[4] + H <= N && ib.numel() == H && fb.numel() == H, "parallel_step: gates");
  TORCH_CHECK(S.dim() == 4 && S.size(0) >= B && S.size(1) == H && S.size(2) == V && S.size(3) == Nq &&
              n.numel() == 2 * S.size(0) * H * Nq && m.numel() == 2 * S.size(0) * H && k_cache.size(0) >= B, "parallel_step: states");
  if (live.has_value()) { check_i(*live, "live"); TORCH_CHECK(live->numel() >= B, "live"); }
  TORCH_CHECK(B < 65536, "parallel_step: rows");
  Tensor q = at::empty({B, attn[3], attn[5]}, k_cache.options()), o = at::empty({B, H * V}, S.options());
  sh.a.q_out = q.data_ptr();
  evgpt::StepMemory sm{rows, (int)mem[0], (int)mem[1], (int)mem[2], (int)mem[3], (int)mem[4], ib.data_ptr<float>(), fb.data_ptr<float>(),
                       (float)cap, (float)qscale, (int)H, (int)Nq, (int)V, S.data_ptr<float>(), n.data_ptr<float>(),
                       m.data_ptr<float>(), (int)S.size(0), o.data_ptr<float>()};
  if (B > 0) evgpt::launch_parallel_step(sh, sm, pos.data_ptr<int>(), iptr(live), f32, (int)B, cur_stream());
  return {q, o};
}
// the state-space recurrence with its convolution and silu(z) gate: [B, H * V] fp32
Tensor ssd_step_(const Tensor& src, at::IntArrayRef dims, const Tensor& conv_w, const Tensor& conv_b, const Tensor& ring,
                 const Tensor& dt_bias, const Tensor& a_log, const Tensor& skip, const Tensor& S, const Tensor& pos, const OptTensor& live) {
  int64_t B, N;
  const SrcRows rows = src_of(src, "src", &B, &N);
  TORCH_CHECK(dims.size() == 7, "ssd_step: {z, x, dt columns, H, G, N, V}");
  const int64_t H = dims[3], G = dims[4], Ns = dims[5], V = dims[6], C = H * V + 2 * G * Ns;
  check_f(conv_w, "conv_w"); check_f(conv_b, "conv_b"); check_t(ring, "ring"); check_f(dt_bias, "dt_bias"); check_f(a_log, "a_log");
  check_f(skip, "skip"); check_f(S, "S"); check_i(pos, "pos");
  TORCH_CHECK(H >= 1 && G >= 1 && H % G == 0 && Ns >= 32 && Ns % 32 == 0 && Ns <= 4096 && (V == 32 || (V >= 64 && V % 64 == 0)), "ssd_step: sizes");
  TORCH_CHECK(dims[0] >= 0 && dims[1] >= 0 && dims[2] >= 0 && dims[0] + H * V <= N && dims[1] + C <= N && dims[2] + H <= N, "ssd_step: sections");
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(0) == C && conv_b.numel() == C && ring.dim() == 3 && ring.size(0) >= B &&
              ring.size(1) == conv_w.size(1) && ring.size(2) == C, "ssd_step: convolution");
  TORCH_CHECK(dt_bias.numel() == H && a_log.numel() == H && skip.numel() == H, "ssd_step: per-head constants");
  TORCH_CHECK(S.dim() == 4 && S.size(0) >= B && S.size(1) == H && S.size(2) == V && S.size(3) == Ns && pos.numel() >= B && B < 65536, "ssd_step: state");
  if (live.has_value()) { check_i(*live, "live"); TORCH_CHECK(live->numel() >= B, "live"); }
  Tensor o = at::empty({B, H * V}, S.options());
  evgpt::StepSsd a{rows, (int)dims[0], (int)dims[1], (int)dims[2], conv_w.data_ptr<float>(), conv_b.data_ptr<float>(), ring.data_ptr(),
                   (int)conv_w.size(1), dt_bias.data_ptr<float>(), a_log.data_ptr<float>(), skip.data_ptr<float>(), (int)H, (int)G,
                   (int)Ns, (int)V, S.data_ptr<float>(), o.data_ptr<float>()};
  if (B > 0) evgpt::launch_ssd_step(a, pos.data_ptr<int>(), iptr(live), is_f32(ring), (int)B, cur_stream());
  return o;
}

// ---------------------------------------------------------------- up to four rows, weights streamed
constexpr int64_t GEMV_LDS = 64 * 1024;
void check_gemv_w(const Tensor& w, int64_t B, int64_t K, const char* name) {
  check_t(w, name);
  TORCH_CHECK(w.dim() == 2 && w.size(1) == K && K % 64 == 0 && K > 0 && w.size(0) % 8 == 0, name, ": [N, K], K % 64 == 0, N % 8 == 0");
  TORCH_CHECK(B >= 1 && B <= evgpt::GEMV_ROWS_MAX, "row_gemv: one to four rows");
}
evgpt::GemvInput stream_input(const Tensor& x, const Tensor& w, int64_t n, double eps, const OptTensor& a, const OptTensor& b,
                              const OptTensor& wa, const OptTensor& wb, const OptTensor& x_out, bool layer) {
  check_stream(x, n); check_f(w, "norm");
  const int64_t K = x.size(1);
  TORCH_CHECK(w.numel() == K, "row_gemv: norm weight size");
  evgpt::GemvInput in{};
  in.kind = evgpt::GV_NORM;
  in.x = x.data_ptr(); in.w = w.data_ptr<float>(); in.n = (int)n; in.eps = (float)eps; in.layer = layer;
  if (a.has_value() && !b.has_value()) {
    TORCH_CHECK(wa.has_value() && x_out.has_value(), "row_gemv: post norm");
    check_f(*a, "a"); check_f(*wa, "wa"); check_f(*x_out, "x_out");
    TORCH_CHECK(a->numel() == x.numel() && wa->numel() == K && x_out->numel() == x.numel() && x_out->data_ptr() != x.data_ptr(),
                "row_gemv: post norm sizes");
    in.kind = evgpt::GV_POST;
    in.a = a->data_ptr<float>(); in.wa = wa->data_ptr<float>(); in.x_out = x_out->data_ptr<float>();
  } else if (a.has_value()) {
    TORCH_CHECK(!layer, "row_gemv: branches are merged with RMS norms");
    TORCH_CHECK(b.has_value() && wa.has_value() && wb.has_value() && x_out.has_value(), "row_gemv: branches");
    check_f(*a, "a"); check_f(*b, "b"); check_f(*wa, "wa"); check_f(*wb, "wb"); check_f(*x_out, "x_out");
    TORCH_CHECK(a->numel() == x.numel() && b->numel() == x.numel() && wa->numel() == K && wb->numel() == K &&
                x_out->numel() == x.numel() && x_out->data_ptr() != x.data_ptr(), "row_gemv: branch sizes");
    in.kind = evgpt::GV_MERGE;
    in.a = a->data_ptr<float>(); in.b = b->data_ptr<float>(); in.wa = wa->data_ptr<float>(); in.wb = wb->data_ptr<float>();
    in.x_out = x_out->data_ptr<float>();
  }
  return in;
}
void run_gemv(const evgpt::GemvCall& c, bool f32, int64_t B) {
  TORCH_CHECK((int64_t)evgpt::row_gemv_lds(c, f32, (int)B) <= GEMV_LDS, "row_gemv: input rows do not fit LDS");
  evgpt::launch_row_gemv(c, f32, (int)B, cur_stream());
}
// W · norm(x): fp32 [B, N], or with act >= 0 act(gate) * up of [gate | up] rows in the storage type.  With branches a, b: x +
// (rms(a) wa + rms(b) wb) / 2 takes x's place and is stored to x_out; with a alone: x + norm(a) wa.  xn_out also gets the
// normed rows.  scale: the fp32 rows are cap * tanh(scale * y / cap) (cap 0: scale * y).
Tensor gemv_norm(const Tensor& x, const Tensor& norm, int64_t n, double eps, const Tensor& w, int64_t act, const OptTensor& a,
                 const OptTensor& b, const OptTensor& wa, const OptTensor& wb, const OptTensor& x_out, bool layer, const OptTensor& xn_out,
                 c10::optional<double> scale, double cap) {
  evgpt::GemvCall c{};
  c.count = 1;
  c.p[0].in = stream_input(x, norm, n, eps, a, b, wa, wb, x_out, layer);
  if (xn_out.has_value()) {
    check_t(*xn_out, "xn_out");
    TORCH_CHECK(xn_out->numel() == x.numel() && xn_out->scalar_type() == w.scalar_type() && c.p[0].in.kind != evgpt::GV_MERGE, "gemv_norm: xn_out");
    c.p[0].in.xn_out = xn_out->data_ptr();
  }
  if (scale.has_value()) {
    TORCH_CHECK(act < 0 && cap >= 0 && c.p[0].in.kind != evgpt::GV_MERGE, "gemv_norm: scaled rows");
    c.finish = 1; c.scale = (float)*scale; c.cap = (float)cap;
  }
  const int64_t B = x.size(0), N = w.size(0);
  check_gemv_w(w, B, x.size(1), "w");
  c.p[0].W = w.data_ptr(); c.p[0].N = (int)N; c.p[0].K = (int)x.size(1);
  Tensor y;
  if (act >= 0) {
    TORCH_CHECK(act == evgpt::GLU_GELU_TANH || act == evgpt::GLU_SILU, "gemv_norm: act 0 or 1");
    y = at::empty({B, N / 2}, w.options());
    c.epilogue = evgpt::GV_GLU; c.h = y.data_ptr(); c.act = (int)act;
  } else {
    y = at::empty({B, N}, x.options());
    c.epilogue = evgpt::GV_STORE; c.p[0].y = y.data_ptr<float>(); c.p[0].ldy = (int)N;
  }
  run_gemv(c, is_f32(w), B);
  return y;
}
// the latent columns of projection rows `src` -> cache [slots, cap, R] at pos (rows whose `live` is 0 are left out)
struct LatentCols { SrcRows s; int64_t rows; };
LatentCols check_latent(const Tensor& src, int64_t col, int64_t n, const Tensor& w, const Tensor& cache, const Tensor& pos,
                        const OptTensor& live, bool f32) {
  LatentCols l;
  int64_t N;
  l.s = src_of(src, "src", &l.rows, &N);
  check_f(w, "latent weight"); check_t(cache, "cache"); check_i(pos, "pos");
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) >= 1 && cache.size(2) % 64 == 0 && cache.size(2) == w.numel() && is_f32(cache) == f32 &&
              n >= 1 && n <= cache.size(2) && col >= 0 && col % 8 == 0 && col + n <= N && pos.numel() >= l.rows, "latent: columns, cache [slots, cap, R]");
  if (live.has_value()) { check_i(*live, "live"); TORCH_CHECK(live->numel() >= l.rows, "latent: live"); }
  return l;
}
// fp32 [B, N] = W · rms(src[:, col .. col + n)); with a cache, the latent columns of the same rows go into it
Tensor gemv_rows(const Tensor& src, int64_t col, int64_t n, const Tensor& norm, double eps, const Tensor& w, int64_t c_col, int64_t c_n,
                 const OptTensor& c_norm, const OptTensor& cache, const OptTensor& pos, const OptTensor& live) {
  int64_t B, cols;
  evgpt::GemvCall c{};
  c.count = 1;
  evgpt::GemvInput& in = c.p[0].in;
  in.kind = evgpt::GV_ROWS;
  in.gate = src_of(src, "src", &B, &cols);
  check_f(norm, "norm");
  const int64_t K = norm.numel(), N = w.size(0);
  TORCH_CHECK(n >= 1 && n <= K && col >= 0 && col % 8 == 0 && col + n <= cols, "gemv_rows: columns");
  check_gemv_w(w, B, K, "w");
  in.gcol = (int)col; in.n = (int)n; in.eps = (float)eps; in.w = norm.data_ptr<float>();
  if (cache.has_value()) {
    TORCH_CHECK(c_norm.has_value() && pos.has_value(), "gemv_rows: latents");
    const LatentCols l = check_latent(src, c_col, c_n, *c_norm, *cache, *pos, live, is_f32(w));
    TORCH_CHECK(cache->size(0) >= B, "gemv_rows: slots");
    c.latent = evgpt::LatentStore{l.s, (int)c_col, (int)c_n, (int)cache->size(2), c_norm->data_ptr<float>(), (float)eps, cache->data_ptr(),
                                  (int)cache->size(1), pos->data_ptr<int>(), iptr(live)};
  }
  Tensor y = at::empty({B, N}, norm.options());
  c.p[0].W = w.data_ptr(); c.p[0].N = (int)N; c.p[0].K = (int)K;
  c.epilogue = evgpt::GV_STORE; c.p[0].y = y.data_ptr<float>(); c.p[0].ldy = (int)N;
  run_gemv(c, is_f32(w), B);
  return y;
}
// fp32 [B, N] = W · h for rows h of the storage type
Tensor gemv_plain(const Tensor& w, const Tensor& h) {
  check_t(h, "h");
  TORCH_CHECK(h.dim() == 2 && h.scalar_type() == w.scalar_type(), "gemv_plain: h [B, K]");
  const int64_t B = h.size(0), N = w.size(0);
  check_gemv_w(w, B, h.size(1), "w");
  Tensor y = at::empty({B, N}, h.options().dtype(at::kFloat));
  evgpt::GemvCall c{};
  c.count = 1;
  c.epilogue = evgpt::GV_STORE;
  c.p[0].W = w.data_ptr(); c.p[0].N = (int)N; c.p[0].K = (int)w.size(1);
  c.p[0].in.kind = evgpt::GV_PLAIN; c.p[0].in.x = h.data_ptr();
  c.p[0].y = y.data_ptr<float>(); c.p[0].ldy = (int)N;
  run_gemv(c, is_f32(w), B);
  return y;
}
// x += W · h for rows h of the storage type
void gemv_add_(const Tensor& x, const Tensor& w, const Tensor& h) {
  check_stream(x, 1); check_t(h, "h");
  const int64_t B = x.size(0);
  TORCH_CHECK(h.dim() == 2 && h.size(0) == B && h.scalar_type() == w.scalar_type() && w.size(0) == x.size(1), "gemv_add: h [B, K], w [width, K]");
  check_gemv_w(w, B, h.size(1), "w");
  evgpt::GemvCall c{};
  c.count = 1;
  c.epilogue = evgpt::GV_ADD;
  c.p[0].W = w.data_ptr(); c.p[0].N = (int)w.size(0); c.p[0].K = (int)w.size(1);
  c.p[0].in.kind = evgpt::GV_PLAIN; c.p[0].in.x = h.data_ptr();
  c.p[0].y = x.data_ptr<float>(); c.p[0].ldy = (int)x.size(1);
  run_gemv(c, is_f32(w), B);
}
evgpt::GemvInput group_input(const Tensor& y, int64_t B, const OptTensor& gate, int64_t gcol, const Tensor& norm, int64_t heads,
                             int64_t v, int64_t vp, int64_t parts, double eps) {
  check_f(y, "y"); check_f(norm, "norm");
  TORCH_CHECK(y.numel() == B * heads * vp && norm.numel() == heads * vp && vp % 8 == 0 && v >= 1 && v <= vp && parts >= 1 &&
              heads * v % parts == 0, "row_gemv: group norm sizes");
  evgpt::GemvInput in{};
  in.kind = evgpt::GV_GROUP;
  in.y = y.data_ptr<float>(); in.w = norm.data_ptr<float>(); in.eps = (float)eps;
  in.heads = (int)heads; in.v = (int)v; in.vp = (int)vp; in.parts = (int)parts;
  if (gate.has_value()) {
    int64_t gm, gn;
    in.gate = src_of(*gate, "gate", &gm, &gn);
    TORCH_CHECK(gm == B && gcol >= 0 && gcol % 8 == 0 && gcol + heads * vp <= gn, "row_gemv: gate columns");
    in.gcol = (int)gcol;
    in.gate_mode = evgpt::GATE_SIGMOID_AFTER;
  }
  return in;
}
// x += W · groupnorm(y)
void gemv_group_add_(const Tensor& x, const Tensor& w, const Tensor& y, const Tensor& norm, int64_t heads, int64_t v, int64_t vp,
                     int64_t parts, double eps) {
  check_stream(x, 1);
  const int64_t B = x.size(0), K = w.size(1);
  TORCH_CHECK(w.size(0) == x.size(1) && K >= heads * vp, "gemv_group_add: w [width, K]");
  check_gemv_w(w, B, K, "w");
  evgpt::GemvCall c{};
  c.count = 1;
  c.epilogue = evgpt::GV_ADD;
  c.p[0].W = w.data_ptr(); c.p[0].N = (int)w.size(0); c.p[0].K = (int)K;
  c.p[0].in = group_input(y, B, c10::nullopt, 0, norm, heads, v, vp, parts, eps);
  c.p[0].y = x.data_ptr<float>(); c.p[0].ldy = (int)x.size(1);
  run_gemv(c, is_f32(w), B);
}
// {Wa · h, Wb · (groupnorm(y) sigmoid(gate))} in one launch: the output projections of an attention branch and a gated
// recurrent branch, fp32 [2, B, width]
Tensor gemv_branches(const Tensor& wa, const Tensor& h, const Tensor& wb, const Tensor& y, const Tensor& gate, int64_t gcol,
                     const Tensor& norm, int64_t heads, int64_t v, int64_t vp, double eps) {
  check_t(h, "h");
  TORCH_CHECK(h.dim() == 2 && h.scalar_type() == wa.scalar_type() && wa.scalar_type() == wb.scalar_type() && wa.size(0) == wb.size(0) &&
              wb.size(1) >= heads * vp, "gemv_branches: h [B, Ka], weights [width, K]");
  const int64_t B = h.size(0), N = wa.size(0);
  check_gemv_w(wa, B, h.size(1), "wa"); check_gemv_w(wb, B, wb.size(1), "wb");
  Tensor o = at::empty({2, B, N}, y.options());
  evgpt::GemvCall c{};
  c.count = 2;
  c.epilogue = evgpt::GV_STORE;
  c.p[0].W = wa.data_ptr(); c.p[0].N = (int)N; c.p[0].K = (int)wa.size(1);
  c.p[0].in.kind = evgpt::GV_PLAIN; c.p[0].in.x = h.data_ptr();
  c.p[0].y = o.data_ptr<float>(); c.p[0].ldy = (int)N;
  c.p[1].W = wb.data_ptr(); c.p[1].N = (int)N; c.p[1].K = (int)wb.size(1);
  c.p[1].in = group_input(y, B, gate, gcol, norm, heads, v, vp, heads, eps);
  c.p[1].y = o.data_ptr<float>() + B * N; c.p[1].ldy = (int)N;
  run_gemv(c, is_f32(wa), B);
  return o;
}

// ---------------------------------------------------------------- latent attention
// Query latents [M, Q] in the storage type (q_norm given) from columns of `src`, key / value latents into `cache` (given)
Tensor latent_prep_(const Tensor& src, int64_t q_col, int64_t nq, const OptTensor& q_norm, int64_t c_col, int64_t nc, const OptTensor& c_norm,
                    const OptTensor& cache, const OptTensor& row_slot, const Tensor& row_pos, const OptTensor& live, double eps, bool f32) {
  int64_t M, N;
  evgpt::LatentPrepArgs a{};
  a.src = src_of(src, "src", &M, &N);
  a.eps = (float)eps;
  check_i(row_pos, "row_pos");
  TORCH_CHECK(row_pos.numel() >= M, "latent_prep: row_pos");
  a.row_pos = row_pos.data_ptr<int>();
  if (row_slot.has_value()) { check_i(*row_slot, "row_slot"); TORCH_CHECK(row_slot->numel() >= M, "latent_prep: row_slot"); a.row_slot = iptr(row_slot); }
  Tensor q;
  if (q_norm.has_value()) {
    check_f(*q_norm, "q_norm");
    const int64_t Q = q_norm->numel();
    TORCH_CHECK(Q % 8 == 0 && nq >= 1 && nq <= Q && q_col >= 0 && q_col % 8 == 0 && q_col + nq <= N, "latent_prep: query columns");
    q = at::empty({M, Q}, q_norm->options().dtype(t_of(f32)));
    a.q_col = (int)q_col; a.nq = (int)nq; a.Q = (int)Q; a.qw = q_norm->data_ptr<float>(); a.q_out = q.data_ptr();
  } else {
    q = at::empty({0}, src.options().dtype(t_of(f32)));
  }
  if (cache.has_value()) {
    TORCH_CHECK(c_norm.has_value(), "latent_prep: c_norm");
    check_latent(src, c_col, nc, *c_norm, *cache, row_pos, live, f32);
    if (!row_slot.has_value()) TORCH_CHECK(cache->size(0) >= M, "latent_prep: slots");
    a.c_col = (int)c_col; a.nc = (int)nc; a.R = (int)cache->size(2); a.cw = c_norm->data_ptr<float>(); a.cache = cache->data_ptr();
    a.cap = (int)cache->size(1); a.live = iptr(live);
  }
  if (M > 0) evgpt::launch_latent_prep(a, f32, (int)M, cur_stream());
  return q;
}
// cached rows into a buffer [rows, R]; copies [n, 4] of {slot, first position, first buffer row, count}
Tensor latent_gather(const Tensor& cache, const Tensor& copies, int64_t rows) {
  check_t(cache, "cache"); check_i(copies, "copies");
  TORCH_CHECK(cache.dim() == 3 && cache.size(2) % 8 == 0 && copies.dim() == 2 && copies.size(1) == 4 && copies.size(0) < 65536 && rows >= 0,
              "latent_gather: cache [slots, cap, R], copies [n, 4]");
  Tensor buf = at::empty({rows, cache.size(2)}, cache.options());
  if (rows > 0 && copies.size(0) > 0)
    evgpt::launch_latent_gather(cache.data_ptr(), buf.data_ptr(), copies.data_ptr<int>(), (int)copies.size(0), is_f32(cache),
                                (int)cache.size(1), (int)cache.size(2), cur_stream());
  return buf;
}
// rows of heads: x [M, H * K] (any SrcRows) -> [M, H, N] in w's type, w [H, N, K]; with a gate, times sigmoid of its column gcol + h
Tensor head_linear(const Tensor& x, const Tensor& w, const OptTensor& gate, int64_t gcol) {
  check_t(w, "w");
  int64_t M, cols;
  evgpt::HeadLinearArgs a{};
  a.x = src_of(x, "x", &M, &cols);
  TORCH_CHECK(w.dim() == 3 && w.size(2) % 64 == 0 && w.size(1) % 64 == 0 && w.size(2) <= 512 && cols >= w.size(0) * w.size(2) &&
              w.size(0) < 65536 && M < 16 * 65535, "head_linear: w [H, N, K]");
  a.w = w.data_ptr(); a.H = (int)w.size(0); a.N = (int)w.size(1); a.K = (int)w.size(2);
  if (gate.has_value()) {
    int64_t gm, gn;
    a.gate = src_of(*gate, "gate", &gm, &gn);
    TORCH_CHECK(gm == M && gcol >= 0 && gcol + a.H <= gn, "head_linear: gate");
    a.gcol = (int)gcol;
  }
  Tensor y = at::empty({M, w.size(0), w.size(1)}, w.options());
  a.y = y.data_ptr();
  if (M > 0) evgpt::launch_head_linear(a, is_f32(w), (int)M, cur_stream());
  return y;
}
// Attention of queries q [M, H, R] in the latent space over positions 0 .. pos[row] of each row's cache, the attended latents
// taken out of it by w_v [H, D, R], heads gated: [M, H, D]
Tensor latent_attend(const Tensor& q, const Tensor& cache, const OptTensor& row_slot, const Tensor& pos, double scale, int64_t nsplit,
                     const Tensor& w_v, const Tensor& gate, int64_t gcol) {
  check_t(q, "q"); check_t(cache, "cache"); check_i(pos, "pos"); check_t(w_v, "w_v");
  const bool f32 = is_f32(q);
  const int64_t M = q.size(0), H = q.size(1), R = q.size(2);
  TORCH_CHECK(q.dim() == 3 && cache.dim() == 3 && cache.size(2) == R && R % 64 == 0 && R <= evgpt::LATENT_MAX && cache.size(1) >= 1 &&
              is_f32(cache) == f32 && is_f32(w_v) == f32 && pos.numel() >= M && M < 65536 && scale > 0, "latent_attend: q [M, H, R], cache [slots, cap, R]");
  if (row_slot.has_value()) { check_i(*row_slot, "row_slot"); TORCH_CHECK(row_slot->numel() >= M, "latent_attend: row_slot"); }
  else TORCH_CHECK(cache.size(0) >= M, "latent_attend: slots");
  TORCH_CHECK(w_v.dim() == 3 && w_v.size(0) == H && w_v.size(1) % 64 == 0 && w_v.size(2) == R, "latent_attend: w_v [H, D, R]");
  if (M == 0) return at::empty({0, H, w_v.size(1)}, q.options());
  const int64_t cap = cache.size(1);
  if (f32) {
    Tensor o = at::empty_like(q);
    evgpt::launch_attn_chunk_decode(q.data_ptr(), cache.data_ptr(), cache.data_ptr(), o.data_ptr(), iptr(row_slot), pos.data_ptr<int>(),
                                    true, (int)M, (int)H, 1, (int)R, (int)cap, (float)scale, cur_stream());
    return head_linear(o.view({M, H * R}), w_v, gate, gcol);
  }
  TORCH_CHECK(R == 64 || R % 128 == 0, "latent_attend: R 64 or a multiple of 128");
  nsplit = std::min<int64_t>(std::max<int64_t>(nsplit, 1), 64);
  Tensor po = at::empty({M, H, nsplit, R}, q.options().dtype(at::kFloat)), pm = at::empty({M, H, nsplit, 2}, q.options().dtype(at::kFloat));
  evgpt::launch_latent_attend(bptr(q), bptr(cache), po.data_ptr<float>(), pm.data_ptr<float>(), iptr(row_slot), pos.data_ptr<int>(), (int)M,
                              (int)H, (int)R, (int)cap, (int)nsplit, (float)scale, cur_stream());
  evgpt::HeadLinearArgs a{};
  int64_t gm, gn;
  a.gate = src_of(gate, "gate", &gm, &gn);
  TORCH_CHECK(gm == M && gcol >= 0 && gcol + H <= gn, "latent_attend: gate");
  a.gcol = (int)gcol;
  a.part_o = po.data_ptr<float>(); a.part_ml = pm.data_ptr<float>(); a.pos = pos.data_ptr<int>(); a.cap = (int)cap; a.nsplit = (int)nsplit;
  a.w = w_v.data_ptr(); a.H = (int)H; a.N = (int)w_v.size(1); a.K = (int)R;
  Tensor y = at::empty({M, H, w_v.size(1)}, q.options());
  a.y = y.data_ptr();
  evgpt::launch_head_linear(a, false, (int)M, cur_stream());
  return y;
}

// ---------------------------------------------------------------- experts
evgpt::MoeRoute route_of(const Tensor& logits, const Tensor& bias, int64_t top, int64_t* rows) {
  int64_t N;
  evgpt::MoeRoute r{};
  r.z = src_of(logits, "router logits", rows, &N);
  check_f(bias, "bias");
  TORCH_CHECK(is_f32(logits) && bias.numel() >= 1 && bias.numel() <= 2048 && N >= bias.numel() && top >= 1 && top <= bias.numel() && top <= 64,
              "router: fp32 logits [M, >= E], up to 2048 experts and 64 chosen");
  r.bias = bias.data_ptr<float>(); r.E = (int)bias.numel(); r.top = (int)top;
  return r;
}
// {experts [M, top], weights [M, top]}
std::tuple<Tensor, Tensor> moe_route(const Tensor& logits, const Tensor& bias, int64_t top) {
  int64_t M;
  const evgpt::MoeRoute r = route_of(logits, bias, top, &M);
  Tensor idx = at::empty({M, top}, bias.options().dtype(at::kInt)), w = at::empty({M, top}, bias.options());
  if (M > 0) evgpt::launch_moe_route(r, idx.data_ptr<int>(), w.data_ptr<float>(), (int)M, cur_stream());
  return {idx, w};
}
// entries of idx [M, top] sorted by expert: {perm, inverse, start [E + 1]}.  idx holds what moe_route wrote: 0 .. E - 1.
std::tuple<Tensor, Tensor, Tensor> moe_group(const Tensor& idx, int64_t E) {
  check_i(idx, "idx");
  TORCH_CHECK(idx.dim() == 2 && E >= 1 && E < 65536 && idx.numel() > 0 && idx.numel() < (1 << 30), "moe_group: idx [M, top]");
  Tensor perm = at::empty({idx.numel()}, idx.options()), inv = at::empty_like(idx), start = at::empty({E + 1}, idx.options());
  evgpt::launch_moe_group(idx.data_ptr<int>(), perm.data_ptr<int>(), inv.data_ptr<int>(), start.data_ptr<int>(), (int)idx.numel(), (int)E, cur_stream());
  return {perm, inv, start};
}
// Rows sorted by expert times each expert's matrix w [E, N, K]: row i is x[perm[i] / top] (gather) or x[i].  act >= 0: w's
// rows are [gate | up] and the result is act(gate) * up [rows, N / 2].
Tensor moe_linear(const Tensor& x, const Tensor& w, const Tensor& start, const OptTensor& perm, int64_t top, int64_t act) {
  check_t(x, "x"); check_t(w, "w"); check_i(start, "start");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && x.scalar_type() == w.scalar_type() && w.size(2) == x.size(1) && start.numel() == w.size(0) + 1,
              "moe_linear: x [M, K], w [E, N, K], start [E + 1]");
  const int64_t E = w.size(0), N = w.size(1), K = w.size(2), A = x.size(0);
  int64_t rows = A;
  if (perm.has_value()) {
    check_i(*perm, "perm");
    rows = perm->numel();
    TORCH_CHECK(top >= 1 && rows == A * top, "moe_linear: perm has top entries per row");
  }
  TORCH_CHECK(rows >= 1 && K % 64 == 0 && K > 0 && N % 64 == 0 && act <= evgpt::GLU_SILU, "moe_linear: K % 64 == 0, N % 64 == 0");
  TORCH_CHECK(A * K < (1ll << 30) && N * K < (1ll << 30) && rows * N < (1ll << 31), "moe_linear: operands are addressed with 32-bit offsets");
  const int* pp = iptr(perm);
  if (is_f32(x)) {
    Tensor y = at::empty({rows, N}, x.options());
    evgpt::launch_gemm_f32_grouped(x.data_ptr<float>(), w.data_ptr<float>(), y.data_ptr<float>(), start.data_ptr<int>(), pp, (int)top,
                                   (int)E, (int)rows, (int)N, (int)K, (int)K, (int)N, cur_stream());
    if (act < 0) return y;
    return glu_rows(y, act, true);
  }
  Tensor y = at::empty({rows, act < 0 ? N : N / 2}, x.options());
  // (the tile's activation: 0 silu, 1 gelu)
  evgpt::launch_gemm_grouped(bptr(x), bptr(w), bptr_mut(y), start.data_ptr<int>(), pp, (int)top, (int)E, (int)A, (int)rows, (int)N, (int)K,
                             act < 0 ? 0 : (act == evgpt::GLU_SILU ? 1 : 2), cur_stream());
  return y;
}
// Up to four rows x [B, K]: fp32 [B, N] = sum_k weight_k Wd_k (act(Wg_k x) * (Wu_k x)) over the chosen experts
Tensor moe_step(const Tensor& x, const Tensor& logits, const Tensor& bias, int64_t top, const Tensor& w_gate_up, const Tensor& w_down, int64_t act) {
  check_t(x, "x"); check_t(w_gate_up, "w_gate_up"); check_t(w_down, "w_down");
  int64_t B;
  evgpt::MoeStep s{};
  s.route = route_of(logits, bias, top, &B);
  const int64_t E = bias.numel(), K = x.size(1), F = w_down.size(2), N = w_down.size(1);
  TORCH_CHECK(x.dim() == 2 && x.size(0) == B && w_gate_up.dim() == 3 && w_down.dim() == 3 && w_gate_up.size(0) == E && w_down.size(0) == E &&
              w_gate_up.size(1) == 2 * F && w_gate_up.size(2) == K && x.scalar_type() == w_gate_up.scalar_type() &&
              x.scalar_type() == w_down.scalar_type() && K % 8 == 0 && F % 8 == 0 && N % 8 == 0 && B >= 1 && B < 65536 &&
              (act == evgpt::GLU_GELU_TANH || act == evgpt::GLU_SILU), "moe_step: x [B, K], w_gate_up [E, 2 F, K], w_down [E, N, F]");
  Tensor h = at::empty({B, top, F}, x.options()), y = at::empty({B, N}, bias.options());
  s.K = (int)K; s.F = (int)F; s.N = (int)N; s.act = (int)act;
  s.x = x.data_ptr(); s.w = w_gate_up.data_ptr(); s.h = h.data_ptr();
  evgpt::launch_moe_step_up(s, is_f32(x), (int)B, cur_stream());
  s.x = h.data_ptr(); s.w = w_down.data_ptr(); s.y = y.data_ptr<float>();
  evgpt::launch_moe_step_down(s, is_f32(x), (int)B, cur_stream());
  return y;
}
int64_t gemv_rows_max() { return evgpt::GEMV_ROWS_MAX; }
int64_t gemv_lds_bytes() { return GEMV_LDS; }

std::tuple<Tensor, Tensor> mlstm_gates(const Tensor& src, int64_t i_col, int64_t f_col, const Tensor& ib, const Tensor& fb, double cap) {
  int64_t M, N;
  const SrcRows s = src_of(src, "src", &M, &N);
  check_f(ib, "ib"); check_f(fb, "fb");
  const int64_t H = ib.numel();
  TORCH_CHECK(fb.numel() == H && i_col >= 0 && f_col >= 0 && i_col + H <= N && f_col + H <= N && cap > 0 && M * H < (1ll << 31), "mlstm_gates: columns");
  Tensor li = at::empty({M, H}, ib.options()), lf = at::empty({M, H}, ib.options());
  if (M > 0)
    evgpt::launch_mlstm_gates(s, (int)i_col, (int)f_col, ib.data_ptr<float>(), fb.data_ptr<float>(), (float)cap,
                              li.data_ptr<float>(), lf.data_ptr<float>(), (int)M, (int)H, cur_stream());
  return {li, lf};
}
std::tuple<Tensor, Tensor> ssd_gates(const Tensor& src, int64_t col, const Tensor& dt_bias, const Tensor& a_log) {
  int64_t M, N;
  const SrcRows s = src_of(src, "src", &M, &N);
  check_f(dt_bias, "dt_bias"); check_f(a_log, "a_log");
  const int64_t H = dt_bias.numel();
  TORCH_CHECK(a_log.numel() == H && col >= 0 && col + H <= N && M * H < (1ll << 31), "ssd_gates: columns");
  Tensor ld = at::empty({M, H}, a_log.options()), dt = at::empty({M, H}, a_log.options());
  if (M > 0)
    evgpt::launch_ssd_gates(s, (int)col, dt_bias.data_ptr<float>(), a_log.data_ptr<float>(), ld.data_ptr<float>(),
                            dt.data_ptr<float>(), (int)M, (int)H, cur_stream());
  return {ld, dt};
}
Tensor conv_rows_(const Tensor& src, int64_t col0, const Tensor& w, const Tensor& bias, const Tensor& ring,
                  const Tensor& row_slot, const Tensor& row_pos, const Tensor& row_first) {
  int64_t M, N;
  const SrcRows s = src_of(src, "src", &M, &N);
  check_f(w, "w"); check_f(bias, "bias"); check_t(ring, "ring"); check_i(row_pos, "row_pos"); check_i(row_slot, "row_slot");
  check_i(row_first, "row_first");
  TORCH_CHECK(w.dim() == 2 && bias.numel() == w.size(0) && ring.dim() == 3 && ring.size(1) == w.size(1) && ring.size(2) == w.size(0),
              "conv_rows: w [C, taps], ring [slots, taps, C]");
  const int64_t C = w.size(0);
  TORCH_CHECK(col0 >= 0 && col0 + C <= N && row_pos.numel() == M && row_slot.numel() == M && row_first.numel() == M, "conv_rows: columns, rows");
  Tensor o = at::empty({M, C}, ring.options());
  if (M > 0)
    evgpt::launch_conv_rows(s, (int)col0, w.data_ptr<float>(), bias.data_ptr<float>(), ring.data_ptr(), o.data_ptr(),
                            is_f32(ring), row_slot.data_ptr<int>(), row_pos.data_ptr<int>(), row_first.data_ptr<int>(), (int)M,
                            (int)C, (int)w.size(1), cur_stream());
  return o;
}
void conv_tail_(const Tensor& src, int64_t col0, const Tensor& ring, const Tensor& tails) {
  int64_t M, N;
  const SrcRows s = src_of(src, "src", &M, &N);
  check_t(ring, "ring"); check_i(tails, "tails");
  TORCH_CHECK(ring.dim() == 3 && tails.dim() == 2 && tails.size(1) == 4 && col0 >= 0 && col0 + ring.size(2) <= N, "conv_tail: shapes");
  if (tails.size(0) > 0)
    evgpt::launch_conv_tail(s, (int)col0, ring.data_ptr(), is_f32(ring), tails.data_ptr<int>(), (int)tails.size(0),
                            (int)ring.size(2), (int)ring.size(1), cur_stream());
}

}  // namespace

TORCH_LIBRARY(evlay, m) {
  m.def("linear(Tensor x, Tensor w, bool out_f32) -> Tensor", &linear);
  m.def("linear_slabs(Tensor x, Tensor w) -> Tensor", &linear_slabs);
  m.def("linear_glu(Tensor x, Tensor w_gate_up, int act) -> Tensor", &linear_glu);
  m.def("embed_rows(Tensor tok, Tensor embed, float scale) -> Tensor", &embed_rows);
  m.def("norm_rows(Tensor x, Tensor? sel, Tensor w, int n, float eps, bool f32, bool layer=False) -> Tensor", &norm_rows);
  m.def("add_norm_rows_(Tensor(a!) x, Tensor y, Tensor? w, int n, float eps, bool f32, bool layer=False) -> Tensor", &add_norm_rows_);
  m.def("post_norm_rows_(Tensor(a!) x, Tensor y, Tensor wy, Tensor? w, int n, float eps, bool f32, bool layer) -> Tensor", &post_norm_rows_);
  m.def("mix_norm_rows_(Tensor(a!) x, Tensor y, Tensor pick, Tensor weights, Tensor? wy, Tensor? w, int n, float eps, bool f32, bool layer) -> Tensor", &mix_norm_rows_);
  m.def("cap_logits_(Tensor(a!) x, float scale, float cap) -> ()", &cap_logits_);
  m.def("gemv_rows(Tensor src, int col, int n, Tensor norm, float eps, Tensor w, int c_col, int c_n, Tensor? c_norm, Tensor(a!)? cache, Tensor? pos, Tensor? live) -> Tensor", &gemv_rows);
  m.def("gemv_plain(Tensor w, Tensor h) -> Tensor", &gemv_plain);
  m.def("latent_prep_(Tensor src, int q_col, int nq, Tensor? q_norm, int c_col, int nc, Tensor? c_norm, Tensor(a!)? cache, Tensor? row_slot, Tensor row_pos, Tensor? live, float eps, bool f32) -> Tensor", &latent_prep_);
  m.def("latent_gather(Tensor cache, Tensor copies, int rows) -> Tensor", &latent_gather);
  m.def("head_linear(Tensor x, Tensor w, Tensor? gate, int gcol) -> Tensor", &head_linear);
  m.def("latent_attend(Tensor q, Tensor cache, Tensor? row_slot, Tensor pos, float scale, int nsplit, Tensor w_v, Tensor gate, int gcol) -> Tensor", &latent_attend);
  m.def("latent_max() -> int", []() { return (int64_t)evgpt::LATENT_MAX; });
  m.def("moe_route(Tensor logits, Tensor bias, int top) -> (Tensor, Tensor)", &moe_route);
  m.def("moe_group(Tensor idx, int E) -> (Tensor, Tensor, Tensor)", &moe_group);
  m.def("moe_linear(Tensor x, Tensor w, Tensor start, Tensor? perm, int top, int act) -> Tensor", &moe_linear);
  m.def("moe_step(Tensor x, Tensor logits, Tensor bias, int top, Tensor w_gate_up, Tensor w_down, int act) -> Tensor", &moe_step);
  m.def("merge_norm_rows_(Tensor(a!) x, Tensor a, Tensor b, Tensor wa, Tensor wb, Tensor? w, int n, float eps, bool f32) -> Tensor", &merge_norm_rows_);
  m.def("glu_rows(Tensor src, int act, bool f32) -> Tensor", &glu_rows);
  m.def("group_norm_rows(Tensor y, Tensor? gate, int gcol, int gate_mode, Tensor w, int heads, int v, int vp, int parts, int ld_out, float eps, bool f32) -> Tensor", &group_norm_rows);
  m.def("commit_rows_(Tensor? logits, Tensor(g!) sampled, Tensor embed, float scale, Tensor(a!) x, Tensor(b!) out_tokens, Tensor(c!) step, Tensor(d!) pos, Tensor(e!) done, Tensor(f!) cur_token, int eos, Tensor? active) -> ()", &commit_rows_);
  m.def("sample_top_p(Tensor logits, Tensor(a!) out, float temperature, float top_p, int seed, Tensor step, int top_k=0) -> ()", &sample_top_p);
  m.def("attn_prep_(Tensor src, int q_col, int k_col, int v_col, Tensor? qw, Tensor? kw, int Hq, int Hkv, int D, int nq, int nk, float eps, Tensor cos, Tensor sin, Tensor? row_slot, Tensor row_pos, Tensor? row_kv, Tensor? row_keep, Tensor(a!)? k_buf, Tensor(b!)? v_buf, Tensor(c!) k_cache, Tensor(d!) v_cache) -> Tensor", &attn_prep_);
  m.def("chunk_keys_copy_(Tensor k_cache, Tensor v_cache, Tensor(a!) k_buf, Tensor(b!) v_buf, Tensor copies) -> ()", &chunk_keys_copy_);
  m.def("attn_chunk(Tensor q, Tensor k, Tensor v, Tensor items, float scale, Tensor? gate=None, int gcol=0) -> Tensor", &attn_chunk);
  m.def("attn_runs_(Tensor q, Tensor k, Tensor v, Tensor(a!) o, int q0, int rows, int kv0, int off, int n, float scale, Tensor? gate=None, int gcol=0) -> ()", &attn_runs_);
  m.def("attn_chunk_decode(Tensor q, Tensor k_cache, Tensor v_cache, Tensor pos, float scale, int nsplit) -> Tensor", &attn_chunk_decode);
  m.def("scan_prefill_(Tensor q, Tensor k, Tensor v, int H, int per_group, int N, int V, float qscale, Tensor log_decay, Tensor? log_in, Tensor? scale_in, Tensor? skip, Tensor(a!) S, Tensor(b!)? n, Tensor(c!)? m, Tensor chunks, Tensor seqs) -> Tensor", &scan_prefill_);
  m.def("parallel_step_(Tensor src, int[] attn, Tensor? qw, Tensor? kw, float eps, Tensor cos, Tensor sin, Tensor(a!) k_cache, Tensor(b!) v_cache, int[] mem, Tensor ib, Tensor fb, float cap, float qscale, Tensor(c!) S, Tensor(d!) n, Tensor(e!) m, Tensor pos, Tensor? live) -> (Tensor, Tensor)", &parallel_step_);
  m.def("ssd_step_(Tensor src, int[] dims, Tensor conv_w, Tensor conv_b, Tensor(a!) ring, Tensor dt_bias, Tensor a_log, Tensor skip, Tensor(b!) S, Tensor pos, Tensor? live) -> Tensor", &ssd_step_);
  m.def("gemv_norm(Tensor x, Tensor norm, int n, float eps, Tensor w, int act, Tensor? a, Tensor? b, Tensor? wa, Tensor? wb, Tensor(a!)? x_out, bool layer=False, Tensor(b!)? xn_out=None, float? scale=None, float cap=0.0) -> Tensor", &gemv_norm);
  m.def("gemv_add_(Tensor(a!) x, Tensor w, Tensor h) -> ()", &gemv_add_);
  m.def("gemv_group_add_(Tensor(a!) x, Tensor w, Tensor y, Tensor norm, int heads, int v, int vp, int parts, float eps) -> ()", &gemv_group_add_);
  m.def("gemv_branches(Tensor wa, Tensor h, Tensor wb, Tensor y, Tensor gate, int gcol, Tensor norm, int heads, int v, int vp, float eps) -> Tensor", &gemv_branches);
  m.def("gemv_blocks(int n) -> ()", [](int64_t n) { evgpt::row_gemv_blocks((int)n); });
  m.def("scan_chunk(bool f32) -> int", [](bool f32) { return (int64_t)(f32 ? evgpt::SCAN_CHUNK_F32 : evgpt::SCAN_CHUNK_BF16); });
  m.def("gemv_rows_max() -> int", &gemv_rows_max);
  m.def("gemv_lds_bytes() -> int", &gemv_lds_bytes);
  m.def("mlstm_gates(Tensor src, int i_col, int f_col, Tensor ib, Tensor fb, float cap) -> (Tensor, Tensor)", &mlstm_gates);
  m.def("ssd_gates(Tensor src, int col, Tensor dt_bias, Tensor a_log) -> (Tensor, Tensor)", &ssd_gates);
  m.def("conv_rows_(Tensor src, int col0, Tensor w, Tensor bias, Tensor ring, Tensor row_slot, Tensor row_pos, Tensor row_first) -> Tensor", &conv_rows_);
  m.def("conv_tail_(Tensor src, int col0, Tensor(a!) ring, Tensor tails) -> ()", &conv_tail_);
}
