// Host-side launcher declarations for every HIP kernel in csrc/kernels.
// Launchers return 0 on success, a hipError_t (>0) on a launch failure, or a
// negative code for an unsupported shape. They never allocate or synchronise,
// so callers may capture them into a hipGraph.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace oamd {
typedef uint16_t bf16_t;

// ---- explanation-model ops ----
int rmsnorm(const bf16_t* x, bf16_t* residual, const bf16_t* w, bf16_t* y, int rows, int hidden,
            int64_t x_stride, int64_t r_stride, int64_t y_stride, float eps, const float* xp, int S,
            hipStream_t stream);
int silu_mul(const bf16_t* gu, bf16_t* out, int64_t rows, int inter, int block, int64_t in_stride,
             int64_t out_stride, int glu, hipStream_t stream);   // glu: Glu of common.h
// Decode-step bookkeeping (norm_act.hip): cache slots + sampler positions of the step's tokens,
// then the state advance after sampling (B <= 1024 rows, one workgroup each).
int decode_slots(const int* bt, const int64_t* pos, const int* ctx, int64_t* slots, int64_t* spos, int B,
                 int max_pages, int page_size, hipStream_t stream);
int decode_advance(const int64_t* tok, int64_t* ids, int64_t* hist, int64_t* pos, int* ctx, int64_t* step, int B,
                   int ms, hipStream_t stream);
int embedding(const int64_t* ids, const bf16_t* table, bf16_t* out, int tokens, int hidden,
              int64_t vocab, hipStream_t stream);
int rope_kv(const bf16_t* qkv, int64_t qkv_stride, const int64_t* pos, const float* cos_t,
            const float* sin_t, int tokens, int Hq, int Hkv, int head_dim, bf16_t* q_out,
            bf16_t* k_out, bf16_t* v_out, void* k_cache, void* v_cache, const int64_t* slots,
            int page_size, int64_t max_pos, const float* xp, int S, const bf16_t* bias,
            bool fp8_cache, float k_scale, float v_scale, hipStream_t stream);  // cache: bf16 or e4m3fn
// Y[M,N] = X[M,K] W[N,K]^T for decode buckets (M a multiple of the BM-row tile, BM in {64,128,256}); S-way split-K
// (S | 8) with fp32 slabs P[S][M][N] reduced into Y; BN in {64, 128} columns per tile.
int gemm_decode(const bf16_t* X, const bf16_t* W, bf16_t* Y, float* P, int M, int N, int K, int S, int BN,
                int BM, int glu, bool w_tiled, int stages, hipStream_t stream);

// Compute-bound 256x256-tile GEMM (prefill projections, lm_head; gemm_tile.hip): Y[M, N] = X[M,K] W[N,K]^T
// (+ bias[N]) for any M >= 1, N % 16 == 0, K % 64 == 0; glu: fused SwiGLU over the 64-row interleaved
// gate|up weight (N % 128 == 0), Y [M, N/2]. ldy = Y's row stride in elements.
// S > 1: S-way split-K into fp32 slabs P[S][M][N], then reduced into Y (SwiGLU applied when glu);
// Y == nullptr leaves the slabs to the consumer (rmsnorm / rope_kv sum them).
int gemm_tile(const bf16_t* X, const bf16_t* W, bf16_t* Y, const bf16_t* bias, int M, int N, int K, int ldy,
              int glu, int variant, int S, float* P, hipStream_t stream);
// Decode-bucket GEMM on the ping-pong schedule (gemm_pp.hip): Y[M,N] = X[M,K] W[N,K]^T, bm-row tiles
// (128 / 256), 128-column tiles (N % 128 == 0), S-way split-K slabs P (S > 1; reduced into Y unless Y is
// nullptr); glu: fused SwiGLU (S == 1), Y [M, N/2]; nt: non-temporal weight loads.
// ws / flags (both given): the stream-K form for bm 256, S 1, nt (gemm_pp.hip SK): ws >= (N / 128) x 32768
// floats, flags >= N / 128 ints, zero (left zero). gemm_pp_sk_grid: its block count, 0 = plain launch.
int gemm_pp(const bf16_t* X, const bf16_t* W, bf16_t* Y, float* P, int M, int N, int K, int S, int bm, int glu,
            bool nt, hipStream_t stream, bool one_seg = false, float* ws = nullptr, int* flags = nullptr);
int gemm_pp_sk_grid(int tiles, int steps);
// 256-row decode GEMM with register-streamed activations (gemm_xr.hip): Xt = X [256, K] in the tiled
// layout [16][K/32][64][8]; N % 128 == 0, K % (64 S) == 0; epi 0 = fp32 slabs P[S][256][N], 1 = bf16 Y,
// 2 = SwiGLU (interleaved gate|up, S == 1) Y [256, N/2], 3 = the same written tiled.
int gemm_xr(const bf16_t* Xt, const bf16_t* W, bf16_t* Y, float* P, int M, int N, int K, int S, int epi,
            hipStream_t stream);
// x [rows, K] row-major -> the tiled layout gemm_xr reads (rows % 16 == 0, K % 32 == 0).
int tile_rows(const bf16_t* x, bf16_t* xt, int rows, int K, hipStream_t stream);
// Y[M, N] = bf16(sum_s P[s][M][N]) (fp32 split-K slabs).
int splitk_reduce(const float* P, bf16_t* Y, int64_t MN, int S, hipStream_t stream);
// Y [M, N/2] = act(gate) * up (glu) of the summed fp32 slabs [S][M][N] of a 64-row interleaved gate|up projection.
int splitk_silu(const float* P, bf16_t* Y, int M, int N, int S, int glu, hipStream_t stream);
// Skinny-M decode GEMM (M <= 32, gemm_skinny.hip): N % 16 == 0, K % (128 S) == 0; S-way split-K slabs P
// reduced into Y (Y == nullptr: left for the consumer); glu: fused SwiGLU over the 64-row
// interleaved gate|up weight, Y [M, N/2].
int gemm_skinny(const bf16_t* X, const bf16_t* W, bf16_t* Y, float* P, int M, int N, int K, int S, int glu,
                hipStream_t stream);

// FP8 e4m3fn W8A8: Y = (X8 . W8^T) * sx[m] * sw[n]; any M (BM-row tiles), S | 8 split-K.
int gemm_fp8(const uint8_t* X, const uint8_t* W, const float* sx, const float* sw, bf16_t* Y, float* P, int M,
             int N, int K, int S, int BN, int BM, hipStream_t stream);
// Per-row dynamic quantization to e4m3fn: sx[m] = max|x[m]| / 448.
int quantize_fp8_rows(const bf16_t* x, uint8_t* q, float* sx, int M, int K, int64_t ld, hipStream_t stream);
// Fused SwiGLU + per-row e4m3fn quantization of the 64-feature-interleaved gate|up rows [M, 2 inter]
// (inter % 64 == 0, <= 16384): q [M, inter], sx [M].
// gu == nullptr: the gate|up rows are the S fp32 split-K slabs P [S, M, 2 inter] (summed, bf16-rounded).
int silu_quantize_fp8(const bf16_t* gu, const float* P, int S, uint8_t* q, float* sx, int M, int inter, int64_t ld,
                      hipStream_t stream);

// Pattern-event scoring + per-doc ranking / summary (N5), see score.hip.
int score_events(const int64_t* keys, const int* hit_doc, const int* doc_ptr, int n_hits, int n_docs,
                 const int* prim_ptr, const int* prim_pat, const int* ev_ptr, const int* ev_doc_ptr,
                 const int* sec_ptr, const int* sec_matcher, const double* sec_w, const int* sec_win,
                 const double* conf, const int* severity, int num_matchers, double significance, double* ev_score,
                 int* ev_pat, int* ev_line, int* order, int* summary, hipStream_t stream);

// The decode step's RoPE + KV-cache write folded into decode attention (rope_kv's decode
// work): q is rotated from the QKV projection inside every workgroup, and the workgroup
// holding a sequence's last token writes that token's rotated K and its V into the cache.
// Row b of the projection is bf16(sum of S fp32 split-K slabs [S][rows][ncol] (+ bias)) or
// a bf16 row (+ bias), ncol = (Hq + 2 Hkv) * 128 -- the numerics of rope_kv.
struct DecRope {
  const float* xp;          // split-K slabs, or nullptr
  const bf16_t* row;        // bf16 rows [rows][row_stride] when xp == nullptr
  int64_t row_stride;
  int S;                    // slab count (xp)
  int64_t slab;             // elements per slab = rows * ncol
  const bf16_t* bias;       // [(Hq + 2 Hkv) * 128] or nullptr
  const int64_t* pos;       // [rows] positions of the decode tokens
  const float* cos_t;       // [max_pos][64]
  const float* sin_t;
  int64_t max_pos;
  const int64_t* slots;     // [rows] cache slot of the decode token (< 0: none)
  float k_inv, v_inv;       // fp8 cache: 1 / k_scale, 1 / v_scale
};

// k_cache / v_cache: bf16, or (fp8) OCP e4m3fn bytes holding x / k_scale, x / v_scale
// rope != nullptr: q is unused; see DecRope
int attn_decode(const bf16_t* q, const void* k_cache, const void* v_cache, bool fp8, float k_scale, float v_scale,
                const int* block_tables, const int* seq_lens, bf16_t* out, float* o_part, float* ml_part, int B,
                int Hq, int Hkv, int head_dim, int page_size, int max_pages, int num_splits, float scale, int variant,
                hipStream_t stream, uint8_t* q8 = nullptr, float* sx = nullptr, const DecRope* rope = nullptr);
// (q8, sx non-null: the output rows are also emitted as per-token e4m3fn [B, Hq*128] + fp32 scales,
// == quantize_fp8_rows(out); `out` then holds valid bf16 only for rows of a single split.)
// Causal prefill attention; the work list holds one item per attn_prefill_block_q(Hq, Hkv, variant)
// query rows of a sequence. variant 1 = per-query-head kernel (64 rows), 2 = GQA-grouped 16-row
// waves, 3 = GQA-grouped swapped-operand 32x32 MFMA waves (2 and 3 need Hq / Hkv in {1, 2, 4, 8}).
int attn_prefill_block_q(int Hq, int Hkv, int variant);
int attn_prefill(const bf16_t* q, const bf16_t* k, const bf16_t* v, bf16_t* o, const int* cu_seqlens,
                 const int* work_seq, const int* work_q0, int num_work, int Hq, int Hkv, int head_dim,
                 float scale, int variant, hipStream_t stream,
                 const bf16_t* pk = nullptr, const bf16_t* pv = nullptr, const int* seq_pfx = nullptr);
int sample_tokens(const void* logits, bool logits_bf16, int64_t stride, int rows, int vocab,
                  const float* temperature, const int64_t* seeds, const int64_t* positions,
                  int64_t* out_tokens, int64_t col_offset, float* out_val, hipStream_t stream);

// One-shot all-reduce over peer-mapped fine-grained buffers (allreduce.hip).
size_t car_buffer_bytes(size_t cap_bytes, int world);
int car_alloc(size_t cap_bytes, int world, void** base, void* handle_out /* 64 B hipIpcMemHandle_t */);
int car_open(const void* handle, void** ptr);
int car_close(void* ptr);
int car_free(void* base);
int car_host_flag(uint32_t** host, uint32_t** dev);   // host-mapped error word (read without a device sync)
void car_free_host_flag(uint32_t* host);
int car_error(const uint32_t* host);
int car_reset(void* base, size_t bytes, uint32_t* host);
// Fused one-shot all-reduce + residual add + RMSNorm (bf16 rows of `hidden`, hidden % 8 == 0, <= 16384):
// residual += bf16(sum over ranks of in); y = rmsnorm(residual) * w. Exactly one of `in` (bf16 rows) and
// `slabs` (S fp32 split-K slabs [S, rows, hidden], summed then bf16-rounded) is non-null; q8/sx non-null
// also emit per-row e4m3fn of y (== quantize_fp8_rows(y)).
// all-reduce protocols (allreduce.hip): one-shot / two-shot (reduce-scatter + all-gather)
// with sc0 sc1 hand-offs, and the original system-fence one-shot (A/B)
constexpr int kCarOneShot = 0, kCarTwoShot = 1, kCarOneShotFence = 2, kCarLL = 3;
int car_all_reduce_rmsnorm(const void* in, const float* slabs, int S, bf16_t* residual, const bf16_t* w, bf16_t* y,
                           uint8_t* q8, float* sx, int rows, int hidden, float eps, int rank, int world,
                           void* const* bases, size_t cap_bytes, int blocks, uint32_t* herr_dev, double timeout_s,
                           int proto, hipStream_t stream);
int car_all_reduce(const void* in, void* out, int64_t bytes, bool bf16, int rank, int world, void* const* bases,
                   size_t cap_bytes, int blocks, uint32_t* herr_dev, double timeout_s, int proto,
                   hipStream_t stream);

// Hyper-connection step over S parallel fp32 residual streams (streams.hip): finishes one
// sublayer (mix [from][to], out) and starts the next (in, norm weight w).
struct StreamStep {
  float* x;                 // [T][S][ld] streams
  int S, width, ld;         // true width and padded row length (ld % 8 == 0)
  const int64_t* ids;       // first step: token ids (streams written from the embedding), else nullptr
  const void* table;        // [vocab][ld], element type of h
  int64_t vocab;
  float emb_scale;
  const float* yp;          // sublayer output as ys fp32 slabs, y_slab elements apart, or
  int ys;
  int64_t y_slab;
  const void* y;            // as rows [T][ld] of h's type (nullptr: none)
  const float* gate;        // [T] logits; sigmoid(gate) scales yp / y (nullptr: 1)
  const void* e;            // rows added on top: row epos[t * top + k] (epos nullptr: t * top + k) of e [.][ld]
  const int* epos;
  int top;                  // 0: none
  const float *mix, *out;   // [S][S], [S] (fp32)
  const float* in;          // [S]
  const float* post_w;      // [ld] norm weight of the sublayer's own output before it joins (one stream), or nullptr
  const float* w;           // [ld] norm weight (fp32, zero past width)
  void* h;                  // [rows][ld] bf16 or fp32
  float eps;
  bool f32;                 // element type of table / y / e / h
  bool sum;                 // last step: u is the plain sum of the streams
  bool write_x;             // write the new streams back
  const int64_t* rows;      // last step: rows to produce (nullptr: all)
};
int stream_step(const StreamStep& a, int n_rows, hipStream_t stream);

// Packed QKV rows -> rotated, per-head-normalised q / k, (mixed) v and the paged cache
// (qkv_heads.hip).
struct QkvHeads {
  const float* xp;          // S fp32 slabs [S][T][ncol], slab elements apart, or nullptr
  int S;
  int64_t slab;
  const void* row;          // [T][ncol] rows (bf16 / fp32)
  int ncol;
  const float* bias;        // [ncol] or nullptr
  const int64_t* pos;
  const float *cos_t, *sin_t;   // [max_pos][rot_ld]
  int rot_pairs, rot_ld;
  int64_t max_pos;
  int Hq, Hkv, dk, dkp, dvp;    // dk: true q/k size (the norm's mean); dkp, dvp: stored sizes
  bool norm;
  float eps;
  const void* v_first;      // [T][Hkv][dvp] or nullptr: v <- (1 - lam) v + lam v_first
  const float* lam;
  void *q_out, *k_out, *v_out;
  void *k_cache, *v_cache;
  const int64_t* slots;     // < 0: not cached
  int log2_page;            // tokens per cache page = 1 << log2_page
};
int qkv_heads(const QkvHeads& a, int tokens, bool f32, hipStream_t stream);

// General-head-size attention, bf16 (attn_gd_prefill.hip, attn_gd_decode.hip)
struct AttnPrefill {
  const bf16_t *q, *k, *v;      // [T][Hq][dkp], [T][Hkv][dkp], [T][Hkv][dvp]
  bf16_t* o;                    // row t, head h at t * o_ld + h * dvp
  int o_ld;
  const int *cu_seqlens, *work_seq, *work_q0;   // work items of 128 query rows
  int Hkv, G, gc, dkp, dvp;     // G query heads per kv head, gc of them (<= 4, divides G) per workgroup
  float scale_log2;
  const bf16_t *pk, *pv;        // shared-prefix rows and per-sequence prefix lengths, or nullptr
  const int* seq_pfx;
  int window;                   // a query sees keys less than this far back (kNoWindow: all)
  const float* gate;            // [T][Hq]: every head's output times its gate, or nullptr
};
constexpr int kNoWindow = 1 << 30;
int attn_gd_prefill(const AttnPrefill& a, int num_work, hipStream_t stream);
struct AttnDecode {
  const bf16_t* q;              // [B][Hq][dkp]
  const bf16_t *k_cache, *v_cache;
  const int *block_tables, *seq_lens;
  bf16_t* out;
  int o_ld;
  float *o_part, *ml_part;      // [B][Hq][num_splits][dvp], [..][2] when num_splits > 1
  int Hkv, G, dkp, dvp, page_size, log2_page, max_pages, num_splits;
  float scale_log2;
  int window;                   // as in AttnPrefill
  const float* gate;            // [B][Hq] or nullptr
};
int attn_gd_decode(const AttnDecode& a, int B, hipStream_t stream);
// Sums the partials of split sequences (split length a multiple of `round` tokens).
int attn_combine(const AttnDecode& a, int B, int round, hipStream_t stream);
// Latent rows (attn_latent_decode.hip): k_cache [pages][P][dkp], values are a row's first rp dims, Hkv = 1,
// G heads, dvp = rp (out and partials rows), dkp % 64 == 0 in 128..640.
int attn_latent_decode(const AttnDecode& a, int B, int rp, hipStream_t stream);

// Short-convolution heads (conv_heads.hip)
struct ConvHeads {
  int T;                    // tokens
  const float* xp;          // S fp32 slabs [S][T][ncol], slab elements apart, or nullptr
  int S;
  int64_t slab;
  const void* row;          // [T][ncol] rows (bf16 / fp32): q | k | gate logits
  int ncol;
  int taps;                 // 1..8
  const void* conv;         // [taps][(Hq + Hkv) dkp], last row: the current token's weight (row type)
  const void *qw, *kw;      // [dkp] norm weights, zero past dk (row type)
  const int64_t* pos;
  int Hq, Hkv, dk, dkp, dvp;
  float eps;
  const int* cu_seqlens;    // prefill: [num_seqs + 1], else nullptr
  int num_seqs;
  const int* prev_page;     // [num_seqs] page of the tokens before a sequence's first row (-1: none), or nullptr
  const int* block_tables;  // decode: [T][max_pages], else nullptr
  int max_pages;
  void* tails;              // [pages][taps - 1][(Hq + Hkv) dkp]
  int64_t pages;
  void *q_out, *k_out, *v_out;   // [T][Hq][dkp], [T][Hkv][dkp], [T][Hkv][dvp] (k_out / v_out may be nullptr)
  void *k_cache, *v_cache;
  const int64_t* slots;     // < 0: not kept
  int log2_page;
  float* gate;              // [T][Hq] sigmoid gates
};
int conv_heads(const ConvHeads& a, bool f32, hipStream_t stream);

// Latent attention (latent.hip)
struct LatentRows {
  const float* xp;          // as in ConvHeads; columns: query latent qp | latent rp | rotated part rotp | gates
  int S;
  int64_t slab;
  const void* row;
  int ncol;
  int q_rank, qp, kv_rank, rp, rot, rotp, ck, H;   // true sizes (the norms' means) and stored ones
  const float *qw, *cw;     // [qp], [rp] norm weights, zero past the true size
  float eps;
  const int64_t* pos;
  const float *cos_t, *sin_t;   // [max_pos][rot_ld]
  int rot_ld;
  int64_t max_pos;
  void* cq;                 // [T][qp]
  void* lat;                // [T][ck] c | rotated part | zeros; nullptr: the layer has none of its own
  void* cache;              // [pages][P][ck] token rows
  const int64_t* slots;
  float* gate;              // [T][H]
};
int latent_rows(const LatentRows& a, int tokens, bool f32, hipStream_t stream);
struct RotateHeads {
  const float* xp;          // S slabs [S][T][H dp] summed into q, or nullptr: q in place
  int S;
  int64_t slab;
  void* q;                  // [T][H][dp]
  const int64_t* pos;
  const float *cos_t, *sin_t;
  int rot_ld;
  int64_t max_pos;
  int H, dp, d, rot;        // rotated: columns d .. d + rot of a head
};
int rotate_heads(const RotateHeads& a, int tokens, bool f32, hipStream_t stream);
struct HeadGemm {
  const bf16_t *X, *W;      // X row m head h at m ldx + h xh; W [H][N][K]
  bf16_t* Y;
  int M, N, K, H;
  int64_t ldx, xh, ldy, yh;
  int pad, x0, nx;          // pad more columns of Y: X's columns x0 .. x0 + nx, then zeros (pad % 16 == 0)
};
int head_gemm(const HeadGemm& a, hipStream_t stream);

// fp32 forms (f32.hip)
int gemm_f32(const float* X, const float* W, float* Y, int M, int N, int K, int ldy, int glu, const int* gtab,
             const float* rscale, hipStream_t stream);
// One product per head: as HeadGemm, without the extra columns.
int head_gemm_f32(const float* X, const float* W, float* Y, int M, int N, int K, int H, int64_t ldx, int64_t xh,
                  int64_t ldy, int64_t yh, hipStream_t stream);
struct AttnF32 {
  const float *q, *k, *v;       // k / v: packed rows, or the paged cache (token rows)
  float* o;
  int o_ld;
  const int *cu_seqlens;        // packed: [num_seqs + 1]
  int num_seqs;
  const int *block_tables, *seq_lens;   // paged
  int Hkv, dkp, dvp, page_size, max_pages;
  int64_t k_ld, v_ld;           // elements between the rows of one head's keys / values in k, v
  float scale;
  const float *pk, *pv;
  const int* seq_pfx;
  int window;                   // as in AttnPrefill
  const float* gate;            // [rows][Hq] or nullptr
};
int attn_f32(const AttnF32& a, int rows, int Hq, bool paged, hipStream_t stream);

// Routed experts (moe.hip)
// Router: logits of E experts (rows 0..E-1 of wr) and, with `gate`, one more row E, in fp32;
// per token the `top` largest, scored by sigmoid.
int moe_route(const bf16_t* h, const bf16_t* wr, int T, int K, int E, int rows_w, int top, int* ids, float* weights,
              float* gate, float* logits, hipStream_t stream);
int moe_topk(const float* logits, int ld, int T, int E, int top, int* ids, float* weights, float* gate,
             hipStream_t stream);
// Expert-sorted row order, every expert's segment padded to bm rows: pos[slot] = row, src[row] =
// token (-1: padding), rscale[row], gtab = {tiles, expert of tile i ...}; slots = T * top.
int moe_sort(const int* ids, const float* weights, int slots, int top, int E, int bm, int max_rows, int* pos, int* src,
             float* rscale, int* gtab, hipStream_t stream);
// xp[row] = h[src[row]] (zeros for padding) for the rows of gtab's tiles; row_bytes % 16 == 0
int moe_gather(const void* h, const int* src, const int* gtab, int bm, int max_rows, void* xp, int row_bytes,
               hipStream_t stream);
// Decode: row slot of Y = X row (slot / div) . W[ids[slot]]^T; glu: SwiGLU of weights[slot] * the
// products over the 64-row interleaved gate|up weight. W [E][N][K], K % 64 == 0, N % 16 == 0 (silu: 128).
int moe_gemm_skinny(const bf16_t* X, const bf16_t* W, bf16_t* Y, const int* ids, const float* weights, int slots,
                    int div, int E, int N, int K, bool silu_gu, hipStream_t stream);
// Row tiles of bm = 64 or 128 sorted rows on the decode GEMM (gemm.hip); src: gathers X rows on the way in.
int moe_gemm_rows(const bf16_t* X, const bf16_t* W, bf16_t* Y, int max_rows, int N, int K, int bm, bool silu_gu,
                  const int* gtab, const int* src, const float* rscale, hipStream_t stream);
// Prefill: rows sorted by moe_sort with bm = 256, persistent 256 x 256 tiles (gemm_tile.hip).
int moe_gemm_tile(const bf16_t* X, const bf16_t* W, bf16_t* Y, int max_rows, int N, int K, bool silu_gu,
                  const int* gtab, const float* rscale, hipStream_t stream);

}  // namespace oamd
