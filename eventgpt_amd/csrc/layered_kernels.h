// Launchers of the layered decoders' kernels (mixers with recurrent state, chunk-masked attention, an
// fp32 residual stream).  As in evgpt_kernels.h they take raw pointers and a stream, allocate nothing
// and never synchronise.  `f32` selects the storage type of weights and activations: float or bf16.
#pragma once
#include <hip/hip_runtime.h>

namespace evgpt {

typedef unsigned short bf16_t;

// Rows produced by a projection: nslab fp32 slabs to be summed, or one matrix of bf16 / fp32.
struct SrcRows {
  const void* p;
  long long slab;   // elements between slabs
  int nslab;
  int ld;           // elements between rows
  int f32;
};

// Rows that are weighted sums of rows of another matrix: row = sum over k < top of w[row][k] * y[pick[row][k]].
struct MixRows {
  const void* y;    // [..][ld], T
  const int* pick;  // [rows][top]
  const float* w;   // [rows][top]
  int top, ld;
};

// ---- gemm_f32.hip
void launch_gemm_f32(const float* A, const float* W, float* C, int M, int N, int K, int lda, int ldw, int ldc,
                     hipStream_t st);

// ---- rowops.hip.  Row widths are padded to a multiple of 64 with zeros (ld); norms divide by the true width n.
enum { GLU_GELU_TANH = 0, GLU_SILU = 1 };
void launch_embed_rows(const int* tok, const void* embed, bool f32, float scale, float* x, int rows, int ld, int vocab,
                       hipStream_t st);
// `layer`: layer norm (mean taken off), otherwise RMS norm.
// xn[i] = norm of x[sel ? sel[i] : i] * w
void launch_norm_rows(const float* x, const int* sel, const float* w, void* xn, bool f32, int rows, int n, int ld,
                      float eps, bool layer, hipStream_t st);
// x += y; xn = norm of x * w (skipped when w is null, here and below)
void launch_add_norm_rows(float* x, const SrcRows& y, const float* w, void* xn, bool f32, int rows, int n, int ld,
                          float eps, bool layer, hipStream_t st);
// x += norm(y) * wy; xn = norm of x * w
void launch_post_norm_rows(float* x, const SrcRows& y, const float* wy, const float* w, void* xn, bool f32, int rows, int n,
                           int ld, float eps, bool layer, hipStream_t st);
// the same with y the weighted sum of picked rows (without wy: x += y)
void launch_mix_norm_rows(float* x, const MixRows& y, const float* wy, const float* w, void* xn, bool f32, int rows, int n,
                          int ld, float eps, bool layer, hipStream_t st);
// x[i] = cap * tanh(scale * x[i] / cap) (cap 0: scale * x[i]); n % 4 == 0
void launch_cap_logits(float* x, long long n, float scale, float cap, hipStream_t st);
// x += (rms(a) * wa + rms(b) * wb) / 2; xn = RMS norm of x * w (skipped when w is null)
void launch_merge_norm_rows(float* x, const SrcRows& a, const SrcRows& b, const float* wa, const float* wb,
                            const float* w, void* xn, bool f32, int rows, int n, int ld, float eps, hipStream_t st);
// h[row][i] = act(src[row][i]) * src[row][ip + i], i < ip
void launch_glu_rows(const SrcRows& src, void* h, bool f32, int rows, int ip, int act, hipStream_t st);
// Group norm of channels stored as heads of vp slots (v of them used): `parts` equal runs of the heads * v true
// channels, each by its own root mean square, times w (laid out like the channels), with a gate read from `gate` at column
// gcol + channel slot: silu(gate) multiplied in before the norm, or sigmoid(gate) after it.
enum { GATE_NONE = 0, GATE_SILU_BEFORE = 1, GATE_SIGMOID_AFTER = 2 };
void launch_group_norm_rows(const SrcRows& y, const SrcRows& gate, int gcol, int mode, const float* w, void* out, bool f32,
                            int rows, int heads, int v, int vp, int parts, int ld_out, float eps, hipStream_t st);
// Commit of one token per sequence: the first maximum of its logits, or sampled[b] when logits is null.  `sampled`
// receives the token either way.
void launch_commit_rows(const float* logits, long long ld_logits, int* sampled, const void* embed, bool f32, float scale, float* x, int* out_tokens,
                        int max_out, int* step, int* pos, int* done, int* cur_token, int eos, int B, int ld, int vocab,
                        const int* active, hipStream_t st);

// Attention inputs from a projection: RMS norm of all q rows / all k rows at once (weights or null), rotary embedding
// of the first `rot` dimensions, q -> q_out rows, k / v -> rows of a key buffer and / or a per-sequence
// cache of `cap` slots that holds the positions of the current chunk (slot = position % cap).
struct AttnPrepArgs {
  SrcRows src;
  int q_col, k_col, v_col;         // columns of the sections in src
  const float* qw;                 // [Hq][D] (zero in the padding) or null: no norm
  const float* kw;
  int Hq, Hkv, D;                  // D: padded head size of q, k and v
  int nq, nk;                      // true widths of the q and k projections (norm divisors)
  float eps;
  const float* cos_tab;            // [max_pos][rot / 2]
  const float* sin_tab;
  int rot, max_pos;
  const int* row_slot;             // [rows] cache slot, or null: the row's index
  const int* row_pos;              // [rows]
  const int* row_kv;               // [rows] row of the key buffer, or null: none
  const int* row_keep;             // [rows] nonzero: also into the cache; null: all rows
  void* q_out;                     // [rows][Hq][D]
  void* k_buf; void* v_buf;        // [kv rows][Hkv][D]
  void* k_cache; void* v_cache;    // [slots][Hkv][cap][D]
  int cap;
};
void launch_attn_prep(const AttnPrepArgs& a, bool f32, int rows, hipStream_t st);
// cached keys of a chunk that a portion continues, into the key buffer: copies [n][4] of
// {slot, first cache slot, key buffer row, count}
void launch_chunk_keys_copy(const void* k_cache, const void* v_cache, void* k_buf, void* v_buf, const int* copies, int n,
                            bool f32, int Hkv, int cap, int D, hipStream_t st);

// ---- attn_chunk.hip (D a multiple of 64, up to 512; any number of query heads per key head)
// items [n][4]: {first query row, query rows (<= 64), key buffer row of the chunk's first key, position of the
// first query within the chunk}
// kld: elements between rows of k and of v; gate: rows of T whose column h gates head h of the output; or null
void launch_attn_chunk(const void* q, const void* k, const void* v, void* o, const int* items, int n_items, bool f32,
                       int Hq, int Hkv, int D, long long kld, float scale, const void* gate, int gate_ld, hipStream_t st);
// keys 0 .. pos % cap of every sequence's cache (row b: cache row_slot[b], or b)
void launch_attn_chunk_decode(const void* q, const void* k_cache, const void* v_cache, void* o, const int* row_slot, const int* pos,
                              bool f32, int B, int Hq, int Hkv, int D, int cap, float scale, hipStream_t st);

// ---- latent.hip: one cached row of R (padded) columns per token, keys and values of all heads linear in it
constexpr int LATENT_MAX = 512;
struct LatentPrepArgs {
  SrcRows src;
  int q_col, nq, Q;                // query latent: first column, true and padded size; q_out null: none
  const float* qw;                 // [Q], zero in the padding
  void* q_out;                     // [rows][Q]
  int c_col, nc, R;                // key / value latent; cache null: none
  const float* cw;                 // [R]
  void* cache;                     // [slots][cap][R]
  int cap;
  const int* row_slot;             // [rows] or null: the row's index
  const int* row_pos;              // [rows]
  const int* live;                 // [rows]: 0 keeps the row out of the cache; or null
  float eps;
};
void launch_latent_prep(const LatentPrepArgs& a, bool f32, int rows, hipStream_t st);
// cached rows into a buffer: copies [n][4] of {slot, first position, first buffer row, count}
void launch_latent_gather(const void* cache, void* buf, const int* copies, int n, bool f32, int cap, int R, hipStream_t st);
// y[row][h][0 .. N) = W[h] x[row][h][0 .. K), times sigmoid(gate[row][gcol + h]) with a gate; K % 32 == 0, N % 16 == 0
struct HeadLinearArgs {
  SrcRows x; int x_col;            // input rows: head h at columns x_col + h * K
  const float* part_o; const float* part_ml;   // or (bf16) the splits of attend, merged: part_o not null
  const int* pos; int cap, nsplit;
  const void* w;                   // [H][N][K]
  SrcRows gate; int gcol;          // gate.p null: none
  void* y;                         // [rows][H][N]
  int H, N, K;
};
void launch_head_linear(const HeadLinearArgs& a, bool f32, int rows, hipStream_t st);
// partial attention of q [rows][H][R] over positions 0 .. pos[row] of the rows' caches: part_o [rows][H][nsplit][R],
// part_ml [rows][H][nsplit][2] (maximum in log2 units, sum).  R: 64, 128, 256, 384 or 512; at most 64 splits
void launch_latent_attend(const bf16_t* q, const bf16_t* cache, float* part_o, float* part_ml, const int* row_slot,
                          const int* pos, int rows, int H, int R, int cap, int nsplit, float scale, hipStream_t st);

// ---- moe.hip
// Router logits [rows][>= E] + bias -> the `top` largest in order (the first of equals) and their softmax weights
struct MoeRoute {
  SrcRows z;
  const float* bias;               // [E]
  int E, top;
};
void launch_moe_route(const MoeRoute& r, int* idx, float* w, int rows, hipStream_t st);      // idx, w [rows][top]
// Entries (row * top + k) sorted by expert: perm [n], its inverse inv [n], start [E + 1]
void launch_moe_group(const int* idx, int* perm, int* inv, int* start, int n, int E, hipStream_t st);
// Up to four rows, weights of the chosen experts streamed: h[b][k] = act(Wg x) * (Wu x), y[b] = sum_k w_k Wd h[b][k].
// w_gate_up [E][2 F][K], w_down [E][N][F]
struct MoeStep {
  MoeRoute route;
  const void* x;                   // up: [B][K]; down: h [B][top][F]
  const void* w;
  void* h;                         // up
  float* y;                        // down: [B][N]
  int K, F, N, act;
};
void launch_moe_step_up(const MoeStep& a, bool f32, int B, hipStream_t st);
void launch_moe_step_down(const MoeStep& a, bool f32, int B, hipStream_t st);
// fp32 grouped product (gemm_f32.hip): row i of expert e's group (rows start[e] .. start[e + 1]) is A row perm[i] / top
// (perm null: i) times W[e] [N][K] -> C row i
void launch_gemm_f32_grouped(const float* A, const float* W, float* C, const int* start, const int* perm, int top, int E,
                             int rows, int N, int K, int lda, int ldc, hipStream_t st);

// ---- linear_scan.hip: S_t = exp(a_t) S_(t-1) + b_t v_t k_t^T per head, y_t = S_t q_t
struct ScanArgs {
  const void* q; const void* k; const void* v;   // [rows][..], T
  long long ldq, ldk, ldv;
  int per_group;                   // heads per q / k head
  int H, N, V;                     // padded sizes: N % 32 == 0, V == 32 or V % 64 == 0
  float qscale;
  const float* log_decay;          // [rows][H]
  const float* log_in;             // [rows][H]: b = exp(log_in), with running maximum and normaliser; or null
  const float* scale_in;           // [rows][H]: b; or null
  const float* skip;               // [H]: y += skip * v; or null
  void* out;                       // [rows][H][V]
  float* S;                        // [slots][H][V][N]
  float* n;                        // [2][slots][H][N], indexed by the parity of the next position
  float* m;                        // [2][slots][H]
  int slots;
};
struct ScanChunks {
  // [C][4]: first row, rows (<= the chunk), slot, flags (bit 0: the sequence's last chunk, bit 1: parity of the next position)
  const int* chunks;
  // [nseq][4]: first chunk, chunks, slot, flags (bit 0: from position 0, bits 1 and 2: parities of start and end)
  const int* seqs;
  int C, nseq;
  float* dS;                       // [C][H][V][N]
  float* dn;                       // [C][H][N]
  double* am; double* fl;          // [C][H]
  float* m0;                       // [C][H]
};
constexpr int SCAN_CHUNK_BF16 = 128, SCAN_CHUNK_F32 = 64;      // tokens per chunk
void launch_scan_prefill(const ScanArgs& a, const ScanChunks& c, bool f32, hipStream_t st);
// log gates of the matrix memory: cap * tanh((x + b) / cap), and the log sigmoid of it for the forget gate
void launch_mlstm_gates(const SrcRows& src, int i_col, int f_col, const float* ib, const float* fb, float cap, float* li,
                        float* lf, int rows, int H, hipStream_t st);
// dt = softplus(x + bias), log decay = -exp(a_log) * dt
void launch_ssd_gates(const SrcRows& src, int col, const float* dt_bias, const float* a_log, float* log_decay, float* dt,
                      int rows, int H, hipStream_t st);

// ---- decode_step.hip: one token per sequence (row b is slot b), straight from the projection's rows
struct StepHeads {                 // attention half: heads of AttnPrepArgs, one block each
  AttnPrepArgs a;
  int on;
};
struct StepMemory {                // matrix memory half
  SrcRows src;
  int q_col, k_col, v_col, i_col, f_col;
  const float* ib; const float* fb;
  float cap, qscale;
  int H, N, V;                     // padded sizes
  float* S; float* n; float* m;    // as in ScanArgs
  int slots;
  float* out;                      // [B][H][V]
};
void launch_parallel_step(const StepHeads& h, const StepMemory& m, const int* pos, const int* live, bool f32, int B,
                          hipStream_t st);
struct StepSsd {
  SrcRows src;
  int z_col, x_col, dt_col;        // x, B and C are consecutive
  const float* conv_w; const float* conv_b;     // [C][taps], [C]
  void* ring;                      // [slots][taps][C], T
  int taps;
  const float* dt_bias; const float* a_log; const float* skip;
  int H, G, N, V;
  float* S;                        // [slots][H][V][N]
  float* out;                      // [B][H][V]: y silu(z)
};
void launch_ssd_step(const StepSsd& a, const int* pos, const int* live, bool f32, int B, hipStream_t st);

// ---- row_gemv.hip: up to four rows, weights streamed once, the input prepared and the output finished in the launch
enum { GV_PLAIN = 0, GV_NORM = 1, GV_MERGE = 2, GV_GROUP = 3, GV_POST = 4, GV_ROWS = 5 };
enum { GV_STORE = 0, GV_ADD = 1, GV_GLU = 2 };
struct GemvInput {
  int kind;
  const void* x;                   // PLAIN: [B][K] of T; NORM, MERGE, POST: the fp32 stream [B][K]
  const float* a; const float* b;  // MERGE: branch outputs [B][K], x + (rms(a) wa + rms(b) wb) / 2; POST: x + norm(a) wa
  const float* wa; const float* wb;
  float* x_out;                    // MERGE, POST: the new stream [B][K]
  void* xn_out;                    // NORM, POST: the normed rows [B][K] of T as well; or null
  const float* w;                  // norm weights [K]
  int n;                           // true width
  float eps;
  int layer;                       // NORM, POST: layer norm
  const float* y;                  // GROUP: [B][heads * vp] fp32
  SrcRows gate;                    // GROUP: the gate's rows; ROWS: the input rows, from column gcol on
  int gcol, gate_mode;
  int heads, v, vp, parts;
};
struct GemvProblem {
  const void* W;                   // [N][K]
  int N, K;
  GemvInput in;
  float* y; int ldy;               // STORE: [B][ldy] fp32; ADD: the stream, accumulated
};
struct LatentStore {               // latent row b = RMS norm of n columns of src -> cache[b][pos[b]], R columns
  SrcRows src;
  int col, n, R;
  const float* w;                  // [R]
  float eps;
  void* cache;                     // [slots][cap][R] of T; null: nothing to do
  int cap;
  const int* pos; const int* live;
};
struct GemvCall {
  LatentStore latent;
  int finish;                      // STORE: y = cap * tanh(scale * y / cap) (cap 0: scale * y)
  float scale, cap;
  GemvProblem p[2];
  int count;                       // problems in this launch (same epilogue)
  int epilogue;
  void* h;                         // GLU: [B][N / 2] of T (W is [gate rows | up rows])
  int act;
};
void row_gemv_blocks(int n);       // workgroups of a launch (0: the default); for tuning runs
constexpr int GEMV_ROWS_MAX = 4;
size_t row_gemv_lds(const GemvCall& c, bool f32, int B);     // bytes of LDS the call needs
void launch_row_gemv(const GemvCall& c, bool f32, int B, hipStream_t st);

// ---- conv1d.hip: causal per-channel convolution + silu; the state is the last inputs in a ring of `taps`
// slots (slot = position % taps)
void launch_conv_rows(const SrcRows& src, int col0, const float* w, const float* bias, void* ring, void* out, bool f32,
                      const int* row_slot, const int* row_pos, const int* row_first, int rows, int C, int taps,
                      hipStream_t st);
// last inputs of every sequence of a prefill into the ring; tails [nseq][4]: {first row, rows, slot, start position}
void launch_conv_tail(const SrcRows& src, int col0, void* ring, bool f32, const int* tails, int nseq, int C, int taps,
                      hipStream_t st);

}  // namespace evgpt
