// Host-side launchers of the gfx950 kernel library.  Every launcher validates the shape
// constraints its kernel relies on, enqueues on the given stream (graph-capture safe: no
// allocation, no synchronisation) and returns a hipError_t value (0 = success).
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

#include <string>
#include <vector>

namespace dab {

inline int div_up_host(int a, int b) { return (a + b - 1) / b; }

// Optional Infinity-Cache warm-up riding on a latency-bound launch (common.h l3_warm): up to two byte
// ranges (16-B multiples) read by ``blocks`` workgroups appended to the kernel's grid.
struct L3Warm {
  const char* ptr[2];
  long bytes[2];
  int blocks;  // 0: off
};

// A projection as its consumers see it: rows of ``ld`` columns, finished (S == 1) or as S split-K slabs ``slab``
// elements apart (proj.h)
struct Proj {
  const void* p;
  int f32;
  int S;
  long slab, ld;
};

// A sigmoid gate of an attention's output: columns ``col`` .. of a projection, one for ``per`` neighbours of the output
struct OutputGate {
  Proj y;
  int col, per;
};

// norm.hip
int rmsnorm(void* out, void* res_out, const void* x, const void* res_in, const void* w, int rows, int cols, float eps,
            hipStream_t s);
int rmsnorm_slabs(void* out, void* res_out, const void* slabs, int S, long slab_stride, const void* res_in,
                  const void* w, int rows, int cols, float eps, hipStream_t s, int slab_bf16 = 0);
int layernorm(void* out, const void* x, const void* res_in, const void* gamma, const void* beta, int rows, int cols,
              float eps, hipStream_t s);
int bert_embed(void* out, const int* ids, const int* pos_ids, const int* type_ids, const void* word, const void* pos,
               const void* type, const void* gamma, const void* beta, int rows, int cols, float eps, hipStream_t s);
int embed_gather(void* out, const int* ids, const void* table, int rows, int cols, hipStream_t s);
int mean_pool(float* out, void* out_bf16, const void* hidden, const int* cu_seqlens, int batch, int cols,
              int normalize, hipStream_t s);

// elementwise.hip
int gelu(void* out, const void* x, const void* bias, size_t rows, int cols, hipStream_t s);
int silu_mul(void* out, const void* x, size_t rows, int F, hipStream_t s, int interleaved = 0);
int rope_kv_write(const void* qkv, int ld, const int* positions, const void* cos_sin, void* q_out, void* k_cache,
                  void* v_cache, const int64_t* slots, int T, int Hq, int Hkv, int D, int block_size, hipStream_t s,
                  const void* slabs = nullptr, int S = 0, long slab_stride = 0, int slab_bf16 = 0);

// attention.hip
int flash_attention(const void* q, long q_stride_tok, long q_stride_head, const void* k, const void* v,
                    long kv_stride_tok, long kv_stride_head, const void* k_cache, const void* v_cache,
                    const int* block_tables, int max_blocks, int block_size, void* out, long o_stride_tok,
                    long o_stride_head, const int* cu_q, const int* cu_k, const int* ctx_k, int batch,
                    int max_seqlen_q, int Hq, int Hkv, int D, int causal, int paged, float scale, hipStream_t s,
                    const int* rope_pos = nullptr, const void* rope_cs = nullptr, int window = 0,
                    const float* sink = nullptr, int chunk = 0, float out_scale = 1.f, const float* slopes = nullptr,
                    const OutputGate* gate = nullptr);  // gate: D = 128, paged, with sink or slopes, over all keys
int paged_decode_attention(const void* q, const void* k_cache, const void* v_cache, const int* block_tables,
                           int max_blocks, int block_size, const int* ctx_lens, void* out, float* part_o,
                           float* part_m, float* part_l, int* counters, int batch, int Hq, int Hkv, int D,
                           int part_size, int max_parts, float scale, hipStream_t s,
                           const int* order = nullptr, const L3Warm* warm = nullptr, int chunk = 0,
                           const float* sink = nullptr, float out_scale = 1.f, long o_stride_tok = 0,
                           const float* slopes = nullptr, const OutputGate* gate = nullptr);

// attention_any.hip (any head width, bf16 or fp32, paged)
int any_attention(const void* q, const void* kc, const void* vc, int f32, const int* bt, int max_blocks, int bs,
                  const int* cu, const int* ctx, int B, int T, int H, int G, int D, int chunk, float scale,
                  const float* sink, const float* slopes, void* out, long o_tok, float out_scale, hipStream_t s);

// rms_stream.hip (RMS norms around an fp32 residual stream; rotary positions and q / k norm before attention)
int rms_residual(float* x, void* h, int act_f32, Proj y, const float* bias, const void* pairs, int top, const int* ids,
                 const void* table, int table_f32, const float* post, const float* gain, int n_true, float eps, int rows,
                 int cols, int fresh, hipStream_t s);
int sigmoid_gate(Proj y, int col0, int per, void* x, long ldx, int act_f32, int n, int T, hipStream_t s);
int softcap(Proj y, float cap, float* out, int n, int T, hipStream_t s);
int qk_rope_write(Proj y, int col0, int H, int G, int D, int dim, int rot, const double* freq, float eps, int norm,
                  const int* positions, const int64_t* slots, void* q, void* kc, void* vc, int act_f32, int bs, int T,
                  hipStream_t s);

// gated_stream.hip (sublayers whose result passes a gate and a norm, sums over depth, PolyNorm)
struct GatedResidual {
  const float* src;          // the stream before (null: zeros)
  float* x;                  // the stream after
  void* h;                   // x, or with ``gain`` its norm, in the activation type
  Proj y;                    // sublayer output (p null: none); row ids[row] with ``ids``
  const int* ids;
  const void* pairs;         // [rows * top, cols] expert rows or null; index >= experts: weight * src instead
  const int* idx;
  const float* wt;
  int top, experts;
  Proj g;                    // gate columns g_col.. (p null: none), their bias
  int g_col;
  const float* g_bias;
  const float* post;         // gain of the norm of what is added
  float* depth;              // n > 0: results 0 .. n - 1, depth_stride apart; keep: x becomes result n
  const float* weights;      // [n + 1]
  long depth_stride;
  int n, keep;
  const float* ahead;        // the sum over results 0 .. from - 1 (null: none, from is 0)
  int from;
  const float* gain;         // or null
  float inv_n, eps;
  int cols;
};
int gated_residual(GatedResidual p, int act_f32, int rows, hipStream_t s);
// out[m] = sum over j < n of w[m][j] result j, for up to 8 rows of w; ``stride`` elements a result
int depth_ahead(const float* over, long stride, const float* w, int n, int m, float* out, hipStream_t s);
int poly_norm(Proj y, int n, int cols, float a, float b, float c, float e, float eps, void* out, int act_f32, int T, hipStream_t s);

// attn_inputs.hip (input projection -> bias, convolution, norm, rotation, temperature, value mix -> q rows and paged cache)
struct AttnInputs {
  Proj y;
  int col0, H, G, D;         // q, k, v heads of D columns from col0
  float inv_q, inv_k, eps;   // 1 / elements of a norm's mean
  int whole;                 // 1: one norm over all q heads and one over all k heads
  const float* gain;         // [(H + G) D]
  const float* bias;         // [(H + 2 G) D] or null
  const float* conv;         // [taps, (H + 2 G) D] or null
  int taps;
  const double* turns;       // turns per position of the rot / 2 pairs
  int rot;
  float rot_mul;             // factor on cosine and sine
  float t_coef;              // query temperature 1 + t_coef ln(floor((p + 1) / t_every) + 1)
  int t_every;
  const int* positions;
  const int64_t* slots;
  void *q, *kc, *vc;         // [T, H, D], caches [blocks, G, bs, D]
  int bs;
  void* ring;                // [slots, taps, (H + 2 G) D]
  const int* slot;           // state slot of every portion / decoded token
  const int* cu;             // portions, or null: decoded tokens from row0
  int row0;
  void* first;               // [T, G, first_w]: mix 1: the values are written here; 2: v += lam (first - v)
  int first_w, mix;
  float lam;
};
int attn_inputs(AttnInputs p, int act_f32, int rows, int max_q, hipStream_t s);

// recurrent.hip (matrix-state recurrences: gated delta rule and state-space duality)
struct RecurrentShape {
  int delta;                       // 1: gated delta rule, 0: state-space duality
  int H, G, D, Dp, V;              // heads, q / k groups, state rows (padded: Dp), value columns
  int C, q_col, k_col, v_col;      // convolution channels and where q, k, v start among them
  int a_col, b_col;                // gate columns (decay / step, beta)
};
int recurrent_state_width(int D);  // D padded as the state is stored
int short_conv(Proj y, int col0, int C, int taps, const float* w, const float* bias, void* ring, const int* slot,
               const int* pos, const int* cu, int chunks, int max_q, void* out, int act_f32, hipStream_t s);
// one decoded token per sequence, rows row0..; with z_out also the C columns z_col.. of the projection as finished rows
int short_conv_step(Proj y, int col0, int C, int taps, const float* w, const float* bias, void* ring, const int* slot,
                    const int* pos, int row0, int B, void* out, int z_col, void* z_out, int act_f32, hipStream_t s);
int state_scan(const void* conv, int act_f32, RecurrentShape d, Proj gates, const float* A, const float* dt_bias,
               const float* skip, float* state, const int* slot, const int* pos, const int* cu, int chunks, void* out,
               hipStream_t s);
// recurrent_chunk.hip: the scan of bf16 portions 64 tokens at a time (prepare + scan); ws: state_chunks_bytes
int state_chunks_ok(RecurrentShape d);
int state_chunks_segments(RecurrentShape d, int chunks, int max_q);
long state_chunks_bytes(RecurrentShape d, int T, int chunks, int segs);
int state_chunks(const void* conv, RecurrentShape d, Proj gates, const float* A, const float* dt_bias, const float* skip,
                 float* state, const int* slot, const int* pos, const int* cu, int chunks, int max_q, int T, int segs, void* out,
                 void* ws, hipStream_t s);
int state_decode(Proj y, int col0, int taps, const float* w, const float* bias, void* ring, int act_f32, RecurrentShape d,
                 Proj gates, const float* A, const float* dt_bias, const float* skip, float* state, const int* slot,
                 const int* pos, int row0, int B, int g_col, const float* norm, float eps, float out_scale, void* out,
                 long ldo, int pad, hipStream_t s);
int gated_norm(const void* y, int act_f32, Proj gate, int g_col, int n, int part, int gate_first, int per_head,
               const float* w, float eps, float scale, void* out, long ldo, int pad, int row0, int T, hipStream_t s);

// selective_scan.hip (diagonal state-space recurrence with a step size, input and read-out of every token)
struct SelectiveShape {
  int C, Np;                 // channels, stored states of a channel (selective_state_width)
  int rank, b_col, c_col;    // columns of the low-rank projection: step [0, rank), input, read-out
  int z_col;                 // gate columns of the input projection
};
int selective_state_width(int N);  // N padded as the state is stored (0: too many)
int narrow_rows(Proj z, float* out, void* low, int N, int R, int T, hipStream_t s);
int selective_scan(const void* u, int act_f32, SelectiveShape d, Proj dt, Proj bc, Proj y, const float* A, const float* dt_bias,
                   const float* skip, float* state, const int* slot, const int* pos, const int* cu, int chunks, int max_q,
                   int segs, float* ws, void* out, hipStream_t s);  // ws (segs > 1): chunks * segs * C * (Np + 1) floats
int selective_segments(SelectiveShape d, int chunks, int max_q);
int selective_step(const void* u, int act_f32, SelectiveShape d, const void* dt_w, const void* low, Proj bc, const float* A,
                   const float* dt_bias, const float* skip, float* state, const int* slot, const int* pos, int row0, int B,
                   void* out, hipStream_t s);

// moe.hip
// scores 0: softmax, weights over their sum; 1: sigmoid scores as they are;
// 2: softmax scores as they are; correction [E] (or null) joins a score where the experts are chosen, not in its weight
int moe_route(Proj z, int col0, int E, int top, float scale, int scores, const float* correction, int* idx, float* wt, int T,
              hipStream_t s);
// pairs whose index is E or more (identity experts) come last in perm and are in no tile
int moe_plan(const int* idx, int P, int E, int bm, int* perm, void* tiles, int max_tiles, int* ws, hipStream_t s);
int moe_plan_words(int P, int E);  // ints of ws (0: none)
int shared_glu(Proj y, int col0, int F, Proj z, int sg_col, void* out, long ldo, int act_f32, int T, hipStream_t s);

// dyt.hip (Dynamic Tanh norms around an fp32 residual stream)
int embed_dyt(float* x, void* h, const int* ids, const void* table, int f32, float scale, float alpha, const float* w,
              const float* b, int rows, int cols, hipStream_t s);
int dyt_residual(float* x, void* h, int h_f32, const void* y, int y_f32, int S, long slab_stride, float a_post,
                 const float* w_post, const float* b_post, const float* ls, float a_next, const float* w_next,
                 const float* b_next, int rows, int cols, hipStream_t s);
int glu_f32(float* out, long ldo, const float* x, long rows, int F, int act, const float* bias, const float* row_scale,
            const int* perm, int scale_in, hipStream_t s);

// gemm_f32.hip (32-bit mode; batched by strides)
int gemm_f32(const float* A, long lda, long sa, const float* B, long ldb, long sb, float* C, long ldc, long sc, int M,
             int N, int K, int batch, hipStream_t s);
// rows of A and C grouped by expert (moe_plan tiles of 64 rows): C[pos] = A[perm[pos] / a_div] . B[expert]^T with
// a_div > 0, A[pos] otherwise; scatter: C row perm[pos]
int gemm_f32_grouped(const float* A, long lda, const float* B, float* C, long ldc, int N, int K, const int* perm, int a_div,
                     int scatter, const void* tiles, int n_tiles, hipStream_t s);

// latent_attention.hip
// rotary positions of latent_write: turns per position of the rot / 2 pairs, factor on cosine and sine, head width of the q
// columns and where its rotated part starts in a head and in the latent row
struct LatentRope {
  const double* freq;
  const int* positions;
  int rot, D, q_at, c_at;
  float mul;
};
int latent_write(const void* y, int y_f32, int S, long slab_stride, long ld, void* q_out, int q_cols, const float* gain,
                 void* cache, int cache_f32, const int64_t* slots, int T, int R, int rank, float eps, LatentRope rope,
                 hipStream_t s);
int latent_gather(void* out, const void* cache, const int* block_tables, int max_blocks, int block_size,
                  const int* cu_k, const int* ctx, int B, int total, int row_bytes, hipStream_t s);
int head_gemm(void* y, long y_tok, long y_head, const void* x, long x_tok, long x_head, const void* w, int row0, int T,
              int H, int N, int K, hipStream_t s);
int latent_key_fill(void* k, long k_tok, int D, const void* rows, int R, int q_at, int c_at, int rot, int H, int T, hipStream_t s);
int latent_decode_ok(int R);
int latent_decode_values(int R);
int latent_decode_groups(int H, int R);
int latent_decode(const void* q, const void* cache, const int* block_tables, int max_blocks, int block_size,
                  const int* ctx_lens, const float* sink, void* out, float* part_o, float* part_ml, int B, int H, int R,
                  int window, int parts, int min_part, float scale, const int* order, hipStream_t s);
int latent_any(void* out, const void* q, const void* cache, int f32, const int* block_tables, int max_blocks,
               int block_size, const int* cu_q, const int* ctx_lens, int B, const float* sink, int T, int H, int R,
               int window, float scale, hipStream_t s);

// gemm.hip
// b_rows > 0: B is an ops.shuffle_weights copy of b_rows (>= N) rows; epilogue 4 / 6 / 7 = SiLU /
// tanh-GELU / ReLU gate over 8-row [gate | up] groups
int gemm_bt(const void* A, long lda, const void* B, long ldb, void* C, long ldc, const void* bias, const void* residual,
            long ldr, int M, int N, int K, int epilogue, int out_f32, const int* row_group, const int* q_group,
            const uint32_t* allow, int allow_words, hipStream_t s, int b_rows = 0, int b_group = 1);
// a narrow fp32 product (router logits, recurrence gates) as S split-K slabs [S][M][N]: tiles of 32 or (tall) 128
// rows, B a shuffle_weights copy
int gemm_narrow(const void* A, long lda, const void* B, float* C, int M, int N, int K, int S, int tall, hipStream_t s);
// experts: like gemm_f32_grouped, bf16, B = per-expert shuffle_weights copies of N rows; glu: SwiGLU over 8-row groups,
// each row times row_scale[pair] (scale_in: gate and up times it, before the activation).  bm: rows of a tile (32, 128 or 256)
int gemm_grouped(const void* A, long lda, const void* B, void* C, long ldc, int N, int K, const int* perm, int a_div,
                 int scatter, const void* tiles, int n_tiles, int bm, int glu, const float* row_scale, int scale_in,
                 hipStream_t s);

// gemm256.hip (large-M prefill / encoder GEMM, 256x256 phased schedule; epilogue 0 none, 1 GELU,
// 2 SwiGLU on [gate 16 | up 16]-interleaved weight rows; bias / residual optional)
int gemm256_ok(int M, int N, int K, long lda, long ldb);
int gemm256_candidates(const void* A, long lda, const void* B, long ldb, int M, int N, int K, const int* row_group,
                       const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx, int cap,
                       hipStream_t s, int b_rows = 0);
// b_shuf: B in the ops.shuffle_weights layout (the decode GEMM's copy); epilogue 4 = SwiGLU over
// 8-row [gate | up] groups
// diagnostic per-tile s_memtime stamps (benchmarks/gemm_stamps.py); returns the grid or -error
int gemm256_candidates_stamped(const void* A, long lda, const void* B, int M, int N, int K, int b_rows,
                               const float* thr, int* cnt, float* cand_val, int* cand_idx, int cap, void* stamps,
                               int stamp_tiles, hipStream_t s);
int gemm256_stamped(const void* A, long lda, const void* B, void* C, const void* bias, const void* residual, int M,
                    int N, int K, int epilogue, int b_shuf, void* stamps, int stamp_tiles, hipStream_t s, int store_aux);
int gemm256(const void* A, long lda, const void* B, long ldb, void* C, long ldc, const void* bias,
            const void* residual, long ldr, int M, int N, int K, int epilogue, hipStream_t s, int b_shuf = 0,
            int b_group = 1);

// gemm_mid.hip (M = 256..4096: mixed serving steps / single prompts; grouped stream-K over the N x K
// plane, 128 x 256 tiles, in-launch last-arriver combine; B in the shuffle_weights layout;
// epilogue 0 none (+ residual) or 4 SwiGLU over 8-row [gate | up] groups)
int gemm_mid_ok(int M, int N, int K, long lda);
long gemm_mid_slab_bytes();
int gemm_mid_counters(int M, int N);
int gemm_mid(const void* A, long lda, const void* B, void* C, long ldc, const void* residual, long ldr, int M, int N,
             int K, int epilogue, void* slabs, long slab_bytes, int* cnt, int n_cnt, hipStream_t s, int variant = 0,
             int b_group = 1);

// stream_gemm.hip (warp-specialised decode GEMM, M <= 256: bf16 / SwiGLU / fp32 split-K slabs; cfg selects
// the tile / ring configuration, stream_gemm_bn(cfg) = weight rows per workgroup)
int stream_gemm(const void* X, long ldx, const void* W, long ldw, void* out, long ldo, const void* residual, long ldr,
                int M, int N, int K, int S, int epilogue, hipStream_t s, int nt_weights, int cfg, float norm_eps = 0.f,
                int slab_bf16 = 0, int w_group = 1);
int stream_gemm_bn(int cfg);
// fp32 (or bf16: slab_bf16) split-K slabs [S][M][N] -> bf16 [M, N] (+ residual)
int slab_reduce(void* out, long ldo, const void* slabs, int S, int M, int N, const void* residual, long ldr,
                hipStream_t s, int slab_bf16 = 0);
// index_scan.hip: persistent scan for 1..64 queries at K <= 1024, 65..96 at K <= 768 (queries staged in
// LDS once), K % 256 == 0
int index_scan_candidates(const void* X, long ldx, const void* W, long ldw, int M, int N, int K, const int* row_group,
                          const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx, int cap,
                          hipStream_t s);
// ... the same scan over a copy of the rows in the shuffle_weights layout (>= round_up(N, 32) rows)
int index_scan_candidates_shuf(const void* X, long ldx, const void* W, int M, int N, int K, const int* row_group,
                               const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx,
                               int cap, hipStream_t s);
int stream_score_candidates(const void* X, long ldx, const void* W, long ldw, int M, int N, int K, const int* row_group,
                            const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx, int cap,
                            hipStream_t s);
int stream_score_candidates_shuf(const void* X, long ldx, const void* W, int M, int N, int K, const int* row_group,
                                 const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx,
                                 int cap, hipStream_t s);
int stream_gemm_max_m(int cfg);
void stream_gemm_set_slice_xcd(int on);
int stream_gemm_slice_xcd();
int stream_gemm_shuffled(int cfg);  // 1: cfg reads weights in the ops.shuffle_weights layout

// select.hip
// Disallowed tokens of the rows with row_flags[r] != 0 (mask bit clear) -> -inf logits, in place
// (JSON-constrained decoding); rows without the flag are untouched.
int mask_logits(void* logits, int logits_f32, long ld, int rows, int vocab, const uint32_t* mask, int words,
                const int* row_flags, hipStream_t s, long mask_ld = 0);
// vocab-parallel sampling (TP): stage 1 on a vocabulary slice, stage 2 on the all-gathered candidates
int sample_candidates(const void* logits, int logits_f32, long ld, int rows, int vocab, int index_base,
                      uint32_t* cand_key, int* cand_idx, int ncand, hipStream_t s);
int sample_merge(const uint32_t* cand_key, const int* cand_idx, int ncand, int rows, int vocab,
                 const float* temperature, const int* top_k, const float* top_p, unsigned long long seed,
                 int64_t* counters, int* out_tokens, hipStream_t s);
int sample_tokens(const void* logits, int logits_f32, long ld, int rows, int vocab, const float* temperature,
                  const int* top_k, const float* top_p, unsigned long long seed, int64_t* counters, int* out_tokens,
                  float* out_logprobs, hipStream_t s);
int topk_rows(const float* scores, long ld, int rows, int n, int k, float* out_vals, int* out_idx, int64_t index_base,
              int64_t* out_idx64, hipStream_t s);

// two-stage variants (chunked across workgroups); workspace = rows * candidates * 8 bytes
int sample_tokens_2stage(const void* logits, int logits_f32, long ld, int rows, int vocab, const float* temperature,
                         const int* top_k, const float* top_p, unsigned long long seed, int64_t* counters,
                         int* out_tokens, void* workspace, size_t workspace_bytes, hipStream_t s);
int topk_rows_2stage(const float* scores, long ld, int rows, int n, int k, float* out_vals, int* out_idx,
                     int64_t index_base, int64_t* out_idx64, void* workspace, size_t workspace_bytes, hipStream_t s);

// gemm.hip: scores >= thr[m] appended per query (exact threshold top-k of the vector index)
int gemm_score_candidates(const void* A, long lda, const void* B, long ldb, int M, int N, int K, const int* row_group,
                          const int* q_group, const float* thr, int* cnt, float* cand_val, int* cand_idx, int cap,
                          hipStream_t s, int b_rows = 0);

// allreduce.hip: one-shot all-reduce over IPC-mapped peer buffers (TP decode on one node)
size_t allreduce_signal_bytes();
// TP decode: this rank's split-K slabs (S > 0) or bf16 partial (S == 0) -> all-reduce -> + residual
// -> RMSNorm, one launch (bitwise slab_reduce + custom_allreduce + rmsnorm)
int custom_allreduce_rmsnorm(const std::vector<uintptr_t>& bases, int rank, const float* slabs, int S,
                             long slab_stride, const void* x, const void* res_in, void* res_out, void* out,
                             const void* w, int rows, int cols, float eps, long half_bytes, long spin_limit,
                             hipStream_t s);
int custom_allreduce(const std::vector<uintptr_t>& bases, int rank, void* data, long nbytes, long half_bytes,
                     long spin_limit, hipStream_t s);
int allreduce_buffer_alloc(long bytes, int uncached, uintptr_t* out);
int allreduce_buffer_free(uintptr_t ptr);
int ipc_get_handle(uintptr_t ptr, std::string* handle);
int ipc_open_handle(const std::string& handle, uintptr_t* out);
int ipc_close_handle(uintptr_t ptr);
int ipc_probe(uintptr_t ptr);
int allreduce_error(uintptr_t base, int clear);
int allreduce_error_async(uintptr_t base, void* host_word, hipStream_t s);

}  // namespace dab
