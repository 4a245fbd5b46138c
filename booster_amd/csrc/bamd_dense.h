// bamd_dense.h — launch interface and argument blocks of the kernels behind the configured layer stacks (bamd_stack.cpp): dense bfloat16 matrices
// (bamd_dense.hip), row-wise mechanisms (bamd_rows.hip), the state-space recurrence (bamd_ssm.hip), latent attention (bamd_latent.hip), attention over cached keys and
// values (bamd_kv.hip), gated linear attention (bamd_gla.hip).
//
// Every kernel exists for two activation types: bfloat16 (matrix operands in bfloat16, 32-bit accumulation) and float (operands in 32-bit as well; weights are
// widened).  Residual stream, norms, scores, decays and states are 32-bit in both.
//
// Packed matrix [rows][K]: 16-row tiles; per tile the K / 32 blocks follow one another, 1 KiB each: lane l of a wave holds row l % 16, columns (l / 16) * 8 .. + 8 —
// the operand layout of v_mfma_f32_16x16x32_bf16, so that one 16-byte load per lane is one contiguous kilobyte and needs no shuffling, in prompts and in decoding.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

enum { BAMD_ACT_BF16 = 0, BAMD_ACT_F32 = 1 };

struct bamd_dense { const uint16_t * w = nullptr; int rows = 0, K = 0; int row_tiles = 0, k_tiles = 0; size_t bytes = 0; };   // rows: outputs (stored: 16 row_tiles); K: stored, 32 k_tiles

// one entry of a batch: n tokens of a sequence.  Row r of the step's token matrix belongs to entry row_entry[r]; its position is pos0 + (r - row0)
struct bamd_entry {
    int32_t seq, row0, n, pos0;
    int32_t par;                   // which half of the double-buffered per-sequence state holds the values in front of this step (the step writes the other half)
    int32_t kbase;                 // prompts: first row of this sequence in the unpacked key / value scratch (a multiple of 64)
};
struct bamd_batch_dev {            // device arrays of a step
    const bamd_entry * ent; const int32_t * row_entry; const int32_t * tokens;
    int n_entries, rows, n_seq;
    const int32_t * pages; int max_pages;          // [n_seq][max_pages] physical page of every 64 positions
};
#define BAMD_PAGE 64

// ---- row-wise mechanisms ------------------------------------------------------------------------------------------------------------------------
// x' = x + norm(y) (y null: x' = x), then what the next sublayer reads:
//   BAMD_NORM_RMS: norm(y) = y / sqrt(mean(y^2) + eps) * g[0]; h = x' + (x'_prev - x') * mu (mu null: h = x'), x'_prev of a sequence's first row in the step is `prev`
//   BAMD_NORM_LAYER: norm(y) = (y - mean) / sqrt(variance + eps) * g[i]; h = the same norm of x' with gain gi[i] (gi null: h = x'); no token shift
enum { BAMD_NORM_RMS = 0, BAMD_NORM_LAYER = 1 };
struct bamd_residual_args {
    const float * x, * y; int ldy, norm; const float * g; float eps;
    const float * mu; float * prev;                // prev: [2][n_seq][E]
    const float * gi;
    float * xo; void * h; int E, ldh;              // xo [rows][E]; h [rows][ldh], zero beyond E (null: not wanted)
};
void bamd_launch_embed_rows(const bamd_batch_dev & b, const uint16_t * embd, const uint16_t * pos, float scale, int E, int V, float * x, hipStream_t s);
void bamd_launch_residual_rows(int act, const bamd_batch_dev & b, const bamd_residual_args & a, hipStream_t s);
// a N(z) + b N(z^2) + c N(z^3) + e with coef = {a, b, c, e}, N = division by the root mean square over the F values
struct bamd_poly_args { const float * z; int ldz; const float * coef; float eps; void * h; int F, ldh; };
void bamd_launch_poly_rows(int act, int rows, const bamd_poly_args & a, hipStream_t s);
// clamped gated unit: g sigmoid(1.702 g) (u + 1) with g = min(gate, limit), u = clamp(up, +-limit).  z rows: 16 gate columns and 16 up columns in turn, 2 ldh in all
struct bamd_glu_args { const float * z; int ldz; float limit; void * h; int ldh; };
void bamd_launch_glu_rows(int act, int rows, const bamd_glu_args & a, hipStream_t s);
#define BAMD_MAX_NORM_GROUPS 512
// root-mean-square norm in `groups` equal parts, times w
struct bamd_group_norm_args { const float * y; int ldy; const float * w; int groups; float eps; void * h; int n, ldh; };
void bamd_launch_group_norm_rows(int act, int rows, const bamd_group_norm_args & a, hipStream_t s);
// h[i] = norm(x' of row want[i]) * gf with x' as above (the model's last norm, of the kind a.norm); xo null
void bamd_launch_final_rows(int act, const bamd_residual_args & a, const int32_t * want, int n_want, const float * gf, hipStream_t s);
// arg-max of n logit rows, as order-preserving keys (ties to the lowest id); keys must be zero, or clear
void bamd_launch_argmax_rows(const float * logits, int n, int V, unsigned long long * keys, bool clear, hipStream_t s);
// greedy loop: token of entry i = the id in keys[i]; appended to out[i * ldo + step]; advance: one position further, state half flipped, keys
// cleared
void bamd_launch_advance(bamd_entry * ent, int32_t * tokens, unsigned long long * keys, int n, int32_t * out, int ldo, int32_t * step, int advance, int V, hipStream_t s);

// ---- dense matrices -------------------------------------------------------------------------------------------------------------------------------
// f32 [rows][ldo] | activation type [rows][ldo] | activation type, transposed [n][ldo] | activation type, the clamped gated unit of alternating 16-row tiles [rows][ldo]
enum { BAMD_OUT_F32 = 0, BAMD_OUT_ACT = 1, BAMD_OUT_ACT_T = 2, BAMD_OUT_GLU = 3 };
int bamd_launch_dense_gemm(int act, const bamd_dense & w, const void * x, int ldx, int rows, void * out, int ldo, int out_kind, hipStream_t s, float limit = 0.f);
// few rows (<= BAMD_MV_ROWS): the weights stream once; out f32 [rows][ldo].  pre: how the operand comes about —
enum { BAMD_PRE_ROWS = 0, BAMD_PRE_RESIDUAL = 1, BAMD_PRE_POLY = 2, BAMD_PRE_GROUP = 3, BAMD_PRE_FINAL = 4, BAMD_PRE_GLU = 5, BAMD_PRE_LAYER = 6 };     // (LAYER: RESIDUAL and FINAL with layer norms, chosen by res.norm); x given | one row, built in front of the product from the argument block
struct bamd_pre_args { bamd_residual_args res; bamd_poly_args poly; bamd_group_norm_args grp; bamd_glu_args glu; const float * gf; const int32_t * want; };
#define BAMD_MV_ROWS 64
int bamd_launch_dense_mv(int act, const bamd_dense & w, int pre, const bamd_batch_dev & b, const bamd_pre_args * p, const void * x, int ldx, int rows, float * out, int ldo, hipStream_t s);
size_t bamd_dense_mv_lds(int act, int K);         // operand bytes of a built row: must stay within BAMD_MV_LDS
#define BAMD_MV_LDS (96 * 1024)

// ---- state-space recurrence ------------------------------------------------------------------------------------------------------------------------
struct bamd_ssm_args {
    const float * in; int ld;                      // rows of the input projection: [z | x | B | C | dt]
    const float * conv, * conv_b, * dt_bias, * A_log, * D;   // conv [channels][taps]
    float * hist;                                  // [2][n_seq][taps - 1][channels]
    float * state;                                 // [n_seq][heads][N][P]
    float * out; int ldo;                          // y * silu(z), before the norm
    float * filtered, * steps;                     // prompts: scratch [rows][channels] and [rows][heads][2]
    int heads, P, N, groups, taps;
};
int bamd_launch_ssm(const bamd_batch_dev & b, const bamd_ssm_args & a, int max_n, hipStream_t s);

// ---- latent attention ------------------------------------------------------------------------------------------------------------------------------
struct bamd_latent_args {
    const float * in; int ld;                      // rows of the fused projection: [q: heads x D | latent: R | gates: heads]
    int q_off, c_off, g_off;
    const float * c_norm; float eps; float scale;
    const float * sink; int gated;                 // sink null: plain softmax
    int heads, D, R, Rp;                           // D: head size class (32, 64, 128, 256; queries, keys and values padded to it); Rp: latent row in the cache
    void * cache;                                  // [pages][BAMD_PAGE][Rp]
    const uint16_t * ukT;                          // decode: per head the packed transpose of the key up-projection [Rp][D]
    bamd_dense uk, uv;
    void * out; int ldo;                           // [rows][ldo], heads x D
};
struct bamd_qtile { int32_t entry, q0; };
void bamd_launch_latent_store(int act, const bamd_batch_dev & b, const bamd_latent_args & a, hipStream_t s);
// prompts: the latents of every entry's sequence, padded to 64 rows, in one matrix [k_rows][Rp]; k_entry: entry of each 64-row block
void bamd_launch_latent_gather(int act, const bamd_batch_dev & b, const bamd_latent_args & a, const int32_t * k_entry, int k_rows, void * dst, hipStream_t s);
int bamd_launch_latent_prompt(int act, const bamd_batch_dev & b, const bamd_latent_args & a, const bamd_qtile * tiles, int n_tiles, const void * k, const void * vt, int ldv, hipStream_t s);
int bamd_latent_prompt_rows(int act, int D);       // query rows per tile
int bamd_latent_max_rank(int act);
// decoding: one row per entry.  qp: absorbed queries [rows][heads padded to 16][Rp]; part_o [rows][hgroups][splits][16][Rp], part_ml [..][16][2]
int bamd_launch_latent_decode(int act, const bamd_batch_dev & b, const bamd_latent_args & a, void * qp, float * part_o, float * part_ml, int splits, hipStream_t s);

// ---- attention over cached keys and values -----------------------------------------------------------------------------------------------------------
// Grouped heads over 64-position pages; position i sees j <= i with i - j < window or j < keep.  Optional: unit-RMS queries and keys, a cap on the scores (cap tanh(s / cap)),
// a bias per distance and head behind it, a gate per head
struct bamd_kv_args {
    const float * in; int ld;                      // rows of the fused projection
    int q_off, k_off, v_off, g_off;                // heads x D | kv_heads x D | kv_heads x D | heads
    int heads, kv_heads, D, dim;                   // D: head size class (32, 64, 128, 256; queries, keys and values padded to it with zeros); dim: size the unit norm counts
    float eps, scale, cap; int unit, gated;        // cap 0: none
    const float * bias; int bias_top;              // [heads][bias_top + 1] by distance, the last for everything farther; null: none
    int window, keep;
    void * kc, * vc;                               // [pages][kv_heads][BAMD_PAGE][D] and, transposed, [pages][kv_heads][D][BAMD_PAGE]
    float out_scale; void * out; int ldo, out_off; // [rows][ldo], heads x D from column out_off on
};
void bamd_launch_kv_store(int act, const bamd_batch_dev & b, const bamd_kv_args & a, const int32_t * k_entry, int k_rows, hipStream_t s);
int bamd_launch_kv_prompt(int act, const bamd_batch_dev & b, const bamd_kv_args & a, const bamd_qtile * tiles, int n_tiles, hipStream_t s);
int bamd_kv_prompt_rows(int act, int D);           // query rows per tile
// most pages a decoded position reads, of `pages` its sequence may hold
int bamd_kv_span(const bamd_kv_args & a, int pages);
// decoding: one row per entry, its own key and value stored as well.  part_o [rows][kv_heads x head groups][splits][16][D], part_ml [..][16][2]
int bamd_launch_kv_decode(int act, const bamd_batch_dev & b, const bamd_kv_args & a, float * part_o, float * part_ml, int splits, hipStream_t s);
int bamd_kv_groups(const bamd_kv_args & a);        // kv_heads x ceil(heads per kv head / 16)
bool bamd_kv_valid(const bamd_kv_args & a);

// ---- gated linear attention -------------------------------------------------------------------------------------------------------------------------
// S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t with alpha = sigmoid(a2 t + b)^(1 / tau) per key channel
struct bamd_gla_args {
    const float * in; int ld;                      // rows of the fused projection
    int q_off, k_off, v_off, t_off;                // heads x Np | heads x Np | heads x Pp | rank
    const uint16_t * a2; const float * a2b;        // bfloat16 [rank][heads x Np], [heads x Np]
    int rank; float inv_tau, q_scale;
    float * state;                                 // [n_seq][heads][Np][Pp]
    float * y; int ldy;                            // [rows][ldy], heads x Pp
    float * alpha, * seg_state, * seg_decay;       // prompts: scratch [rows][heads x Np], [segments][heads][Np][Pp], [segments][heads][Np]
    int heads, Np, Pp;                             // channels and columns per head, padded to a multiple of four
    // what reads y: per head y / sqrt(mean(y^2) + eps) * norm, times silu of the gate
    int g_off, P; const float * norm; float eps;   // heads x Pp of the projection (-1: no gate); columns the mean counts; [Pp], zero beyond P
    void * out; int ldo, out_off, out_cols;        // [rows][ldo], heads x Pp from column out_off on, zero up to out_cols
};
// a prompt portion is scanned in segments: the states at their starts come from a first scan of every segment alone
struct bamd_segment { int32_t entry, t0, n, first, last; };       // first, last: of the entry's segments
// segs == n_entries: every entry is one segment.  max_n: most tokens any entry brings
int bamd_launch_gla(const bamd_batch_dev & b, const bamd_gla_args & a, int max_n, const bamd_segment * segs, int n_segs, hipStream_t s);
void bamd_launch_gla_norm(int act, const bamd_gla_args & a, int rows, hipStream_t s);
int bamd_gla_blocks(int heads, int Pp);            // blocks of one segment
bool bamd_gla_valid(const bamd_gla_args & a);

// ---- both at once ------------------------------------------------------------------------------------------------------------------------------------
// a decoded token through attention and gated linear attention that read the same projection: their blocks share two launches
int bamd_launch_kv_gla_decode(int act, const bamd_batch_dev & b, const bamd_kv_args & kv, const bamd_gla_args & gla, float * part_o, float * part_ml, int splits, hipStream_t s);
