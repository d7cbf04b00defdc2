/*
 * kf_rb.h -- C ABI of libkf_hip.so, continued: the ROW-BATCH operators.  A row batch is the next tokens of several sequences side by side (prompts of unequal
 * length without padding, or one token of each), every row with its own position and state slot.  The operators work on a 32-bit residual stream, take the kind of
 * every mechanism (activation, chunk size, rotation, gate, scale, experts ...) as a parameter and exist in two storages: KF_BF16 (bf16 operands, 32-bit accumulation)
 * and KF_F32 (true 32-bit throughout).  Conventions of kf_abi.h apply: device pointers, a stream of one ctx, 0 or a negative code, no allocation.
 *
 * Weights of a product in bf16 are stored as MFMA operands: tiles of 16 rows x 32 columns, 1 KB each, in row-of-tiles order; inside a tile the 16-byte piece of row r, columns
 * 8 q .. 8 q + 7 (q < 4) is number 16 q + r -- a wave reads a tile as one contiguous kilobyte, whichever lane it hands a piece to.  fp32 weights stay row-major.
 *
 * Padding: the widths a product runs over are padded with zeros to multiples of KF_RB_PAD in weights and activations alike, weight rows too: tile kernels need no tails.
 */
#ifndef KF_RB_H
#define KF_RB_H
#include "kf_abi.h"

#ifdef __cplusplus
extern "C" {
#endif

#define KF_RB_PAD 64
#define KF_RB_NORM_ROWS 4
#define KF_RB_SUM_PAIRS 1024 /* (row, choice) pairs of a batch the SUM mode takes */
#define KF_RB_DECODE_MAX 64 /* rows of a decode batch the streaming products serve; larger batches take the tile kernels */

/* activations; GELU in its tanh form, as kf_gelu */
enum kf_rb_act { KF_RB_RELU = 0, KF_RB_SILU = 1, KF_RB_GELU_TANH = 2 };

/* what a product's epilogue does with row dot d[t][m]:
 *   STORE      y[t][m] = d             (y in the batch's storage; columns act_lo <= m < act_hi: act(d))
 *   STORE_F32  y[t][m] = d             (fp32)
 *   RESIDUAL   y[t][m] = alpha res[t][m] + d   (fp32)
 *   GATED      y[t][f] = act(d[t][gate f]) * d[t][up f]; the weight holds gate and up interleaved in blocks of 16 rows (16 gate, 16 up, ...), m counts both */
enum kf_rb_epilogue { KF_RB_STORE = 0, KF_RB_STORE_F32 = 1, KF_RB_RESIDUAL = 2, KF_RB_GATED = 3 };

/* the routed (row, choice) pairs of a batch, grouped by expert; pair p = row * top + choice */
typedef struct kf_rb_experts {
    int32_t n_expert, top;
    int32_t tile;               /* pairs per tile of the list (every tile belongs to one expert) */
    int32_t n_tile;             /* tiles the list has room for: kf_rb_list_tiles() */
    const int32_t* tile_expert; /* [n_tile] the tile's expert, -1: empty (a run of them at the end) */
    const int32_t* list;        /* [n_tile][tile] pairs, -1: none */
    const int32_t* ids;         /* [rows * top] chosen expert of every pair, -1: inactive row */
    const float* weight;        /* [rows * top] */
    int64_t w_stride;           /* elements from one expert's matrix to the next */
} kf_rb_experts;

/* how a product meets the experts:
 *   ALL   no experts
 *   UP    pair p reads row p / top of x and writes row p of y; GATED only: y is scaled by the pair's weight before it is stored
 *   DOWN  pair p reads row p of x and writes row p of y (STORE)
 *   SUM   row t: RESIDUAL with d = the sum over its pairs of (expert's matrix . row p of x) -- decode batches only */
enum kf_rb_experts_mode { KF_RB_ALL = 0, KF_RB_UP = 1, KF_RB_DOWN = 2, KF_RB_SUM = 3 };

typedef struct kf_rb_product {
    const void* w;   /* [m][k] (x n_expert), bf16: in tiles */
    const void* x;   /* rows ldx apart */
    void* y;         /* rows ldy apart */
    const float* res;
    int64_t ldx, ldy, ldr;
    int32_t type;    /* KF_BF16 | KF_F32: w, x and a STORE / GATED y */
    int32_t m, k, n; /* m, k: multiples of KF_RB_PAD; n: token rows of the batch.  bf16 with experts: tiles of 16, 32, 48 or 64 pairs (n <= KF_RB_DECODE_MAX), 64 or 128
                        (more rows); fp32: 64 */
    int32_t epilogue, act, mode;
    float alpha;
    const kf_rb_experts* experts;
    /* The norm between two products of a decode batch inside the second (where kf_rb_linear_norms() says 1):
     *   ssq != NULL (RESIDUAL): the sums of squares of y's columns 16 i .. 16 i + 15 go to ssq[i][KF_RB_NORM_ROWS] (row t in column t)
     *   norm_z != NULL (mode ALL): x is FIRST formed as the RMS norm (norm_w, norm_eps, norm_dim columns; pad columns of norm_z and norm_w zero) of the fp32 rows norm_z --
     *     rows ldx = k apart, like x, their sums of squares in norm_ssq -- and left in x (bf16) and norm_x (fp32): kf_rb_norm and the product in one */
    float* ssq;
    const float* norm_z;
    const float* norm_ssq;
    const void* norm_w;
    float* norm_x;
    float norm_eps;
    int32_t norm_dim;
    int32_t act_lo, act_hi; /* STORE: the columns that pass through act; equal: none */
} kf_rb_product;
int kf_rb_linear(kf_ctx* ctx, const kf_rb_product* p);
int kf_rb_linear_norms(int type, int n, int k);

/* load time: a bf16 matrix src [rows][cols] into rows row0 .. of a padded one (ld columns; columns cols .. ld - 1 are left alone: allocate zeroed) of storage `type`.
 * half < 0: row r goes to row row0 + r; half 0 / 1: to row 32 (r / 16) + 16 half + r % 16, the gate / up halves of a GATED product's weight.  tiled (bf16): a product's
 * weight; otherwise row-major (embedding tables, norm weights) */
int kf_rb_pack(kf_ctx* ctx, int type, const kf_bf16* src, int rows, int cols, void* dst, int64_t ld, int row0, int half, int tiled);

/* tokens -> rows of the table: x fp32 [n][ldx] and h (storage `type`) [n][ldx]; columns dim .. ldx - 1 are written as zeros.  table rows are ldx apart too. */
int kf_rb_embed(kf_ctx* ctx, int type, const void* table, int vocab, int dim, int64_t ldx, const int32_t* tokens, int n, float* x, void* h);
/* a decode batch: row s is slot s of a state array d_state [n][4] = {token, pos, parked, status}, token = d_forced[s][pos] when that is >= 0.  Also writes the rows'
 * meta (below); a parked slot, or one whose position is outside [0, max_pos), becomes an inactive row (the latter with status bit 64). */
int kf_rb_embed_state(kf_ctx* ctx, int type, const void* table, int vocab, int dim, int64_t ldx, int32_t* d_state, const int32_t* d_forced, int forced_stride, int max_pos,
                      int n, float* x, void* h, int32_t* meta);

/* RMS norm of fp32 rows, z / sqrt(mean(z^2) + eps) * w over `dim` columns: x_out (fp32, may be NULL) and h_out (storage `type`) both ld apart, pad columns zero.
 *   plain:   z = row t of z
 *   experts: alpha res[t] + sum over the row's `top` pairs of row t * top + j of z, which is in storage `type` then      (res != NULL)
 *   rows != NULL: output row t comes from row rows[t] */
int kf_rb_norm(kf_ctx* ctx, int type, const void* z, const float* res, float alpha, int top, const void* w, float eps, int dim, int64_t ld, int n, const int32_t* rows,
               float* x_out, void* h_out);

/* the norm of a sublayer's OUTPUT, added to the residual, and the norm of an input that takes a position vector first: rows z (fp32, ld apart)
 *   z += the sinusoid of the row's position (pos_hi != NULL; kf_rb_sinusoid_tables_host, position in meta)
 *   n  = the norm of z over `dim` columns, times w:  RMS  z / sqrt(mean(z^2) + eps),  LAYER  (z - mean) / sqrt(mean((z - mean)^2) + eps)
 *   x_out (fp32, may be NULL) and h_out (storage `type`, may be NULL): add + n (add NULL: n), pad columns zero
 * rows != NULL: output row t comes from row rows[t] of z.  In place on z or add is fine without `rows`. */
enum kf_rb_norm_kind { KF_RB_RMS = 0, KF_RB_LAYER = 1 };
typedef struct kf_rb_norming {
    const float* z;
    const float* add;
    const int32_t* rows;
    const void* w; /* [dim], padded to ld, in storage `type` */
    float* x_out;
    void* h_out;
    const float *pos_hi, *pos_lo;
    const int32_t* meta;
    int64_t ld;
    int32_t type, kind, dim, n;
    float eps;
} kf_rb_norming;
int kf_rb_norm_rows(kf_ctx* ctx, const kf_rb_norming* a);
/* host: (sin, cos) of p * base^(-2 i / width) for column pair i, as two factors of the angle: hi [(n_pos + 63) / 64][ld / 2][2] at p = 64 j, lo [64][ld / 2][2]; column 2 i of
 * a position vector is the sine, 2 i + 1 the cosine */
int kf_rb_sinusoid_tables_host(float* hi, float* lo, int n_pos, int width, int64_t ld, double base);

/* a row's meta: {position (< 0: inactive), slot, position of the sequence's first row in this batch, position of its last row in this batch} */
#define KF_RB_META 4
/* a sequence's rows: {first row, rows, position of the first row, slot} */

/* one attention layer over a row batch.  raw [rows][ldraw] holds q (n_head * dim columns), then k (n_kv * dim), then the output gate (n_head * dim, gated != 0).
 * There is no v: a row's value is its k column block as the projection left it.  q and k: RMS norm per head, then the leading rot_dims dimensions turned by the table
 * `rope`, dimension i together with i + rot_dims / 2.  Scores are scale * <q, k>; with chunk > 0 a query sees only its own chunk (positions c chunk .. (c + 1) chunk - 1) up to
 * itself, with chunk 0 everything up to itself.  out [rows][ldout], columns n_head * dim: softmax-weighted values, times sigmoid(gate) when gated.
 * Variants (zero: the form above):
 *   v_col   values are raw columns v_col .. v_col + n_kv * vdim - 1, `vdim` per head; the output gate then starts at column gate_col
 *   unit    q and k are divided by their root mean square, no weight (q_norm = k_norm = NULL)
 *   window  position i sees j with 0 <= i - j < window (chunk 0)
 *   sink    one more score of 0 in the softmax's denominator, without a value
 *   scaled  the output is multiplied by out_scale
 * The state: kv-head g's key (normed, rotated) and value of position j in slot s lie at cache[s * slot_stride + g * head_stride + (j % cache_rows) * dim];
 * cache_rows >= min(chunk, positions).  scratch holds arrival counters: zero it once after allocation. */
typedef struct kf_rb_attention {
    void* raw;
    void* out;
    void* k_new;            /* [rows][n_kv * dim] scratch: the batch's normed, rotated keys (prefill form) */
    void *k_cache, *v_cache;
    const void *q_norm, *k_norm; /* [dim], NULL: no norm */
    const float* rope;      /* [max_pos][rot_dims / 2][2] (cos, sin); rot_dims 0: not read */
    void* scratch;          /* decode form, kf_rb_attention_scratch() bytes */
    int64_t ldraw, ldout, slot_stride, head_stride;
    int32_t type, n_head, n_kv, dim, rot_dims, chunk, cache_rows, gated;
    float scale, eps;
    int32_t v_col, vdim, gate_col, unit, window, sink, scaled;
    float out_scale;
} kf_rb_attention;
/* rows of n_seq sequences, longest max_n rows: seqs [n_seq][4], meta [n_rows][4] on the device */
int kf_rb_attention_prefill(kf_ctx* ctx, const kf_rb_attention* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n);
/* one row per slot; max_pos bounds the positions of the active rows (launch geometry) */
int kf_rb_attention_decode(kf_ctx* ctx, const kf_rb_attention* a, const int32_t* meta, int n_rows, int max_pos);
size_t kf_rb_attention_scratch(int n_rows, int n_head, int dim);
/* host: (cos, sin) of pos * w_i for i < dims / 2, w_i = base^(-2 i / dims) * (t + (1 - t) / factor), t = clamp((original w / 2 pi - low) / (high - low), 0, 1) of the
 * unscaled w: frequencies that turn more than `high` times over `original` positions stay, those below `low` turns slow down by `factor`, a linear blend between. */
int kf_rb_rope_table_host(float* h_table, int n_pos, int dims, double base, double factor, double low, double high, double original);

/* ---- recurrent layers: a 32-bit state matrix S [dim][vdim] per head and slot, carried from row to row
 * state: head h of slot s at state[((s * 2 + side) * n_head + h) * dim * vs], rows of vs = vdim rounded up to 4 floats.  The state AFTER position p lies on side p & 1: a step reads
 * side (p - 1) & 1 and writes the other one, so a step that is run twice on the same position gives the same.  Position 0 starts from zero whatever the slot holds.
 *
 * The gated delta rule with one decay per head and key channel.  raw [rows][ldraw] holds, as projected: q (n_kv * dim) from column 0, k (n_kv * dim), v (n_head * vdim), and from columns
 * col_b: n_head logits of the step sizes, col_a: rank_a, col_g: rank_g inputs of the low-rank factors.  q, k, v: causal convolution over time per channel (conv [channels][taps], last
 * tap the row itself, nothing before position 0), SiLU; q and k per head divided by sqrt(sum of squares + unit_eps), q times q_scale.  Head h uses q / k head h / (n_head / n_kv).
 *   beta = sigmoid(b),  decay g = exp(-exp(a_log[h]) softplus(a + dt_bias)) with a = w_a2 . (rank_a columns), [n_head][dim]
 *   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
 *   out = o / sqrt(mean over vdim (o^2) + eps) * norm_w * sigmoid(w_g2 . (rank_g columns)), [n_head][vdim]
 * hist: the convolution's last inputs, raw columns 0 .. channels - 1 of position p at hist[s * hist_slot + (p % taps) * channels].
 * w_a2 / w_g2 are products' weights of ld_a / ld_g columns; the prompt form takes their products from the caller: a_z fp32 [rows][ld_az], g_z (storage) [rows][ld_gz]. */
typedef struct kf_rb_delta {
    const void* raw;
    void* out;
    const void *conv, *w_a2, *w_g2, *a_log, *dt_bias, *norm_w;
    const float* a_z;
    const void* g_z;
    float* state;
    void* hist;
    float* scratch; /* prompt form: kf_rb_delta_scratch() bytes */
    int64_t ldraw, ldout, ld_az, ld_gz, hist_slot;
    int32_t type, n_head, n_kv, dim, vdim, taps, col_b, col_a, col_g, rank_a, rank_g, ld_a, ld_g;
    float q_scale, unit_eps, eps;
} kf_rb_delta;
int kf_rb_delta_prefill(kf_ctx* ctx, const kf_rb_delta* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n);
int kf_rb_delta_decode(kf_ctx* ctx, const kf_rb_delta* a, const int32_t* meta, int n_rows);
size_t kf_rb_delta_scratch(int type, int n_rows, int n_seq, int n_head, int n_kv, int dim, int vdim);

/* A sum with one constant decay per head: S <- decay[h] S + k v^T, o = S^T q.  raw holds q (n_head * dim) from column col_q, k behind it, v (n_head * vdim) behind that -- activated
 * already -- and from col_g n_head * vdim gate logits.  All heads together: out = out_scale * o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate). */
typedef struct kf_rb_decay {
    const void* raw;
    void* out;
    const void* norm_w;   /* [n_head * vdim] */
    const float* decay;   /* [n_head] on the device */
    float* state;
    float* scratch;       /* kf_rb_decay_scratch() bytes, zeroed once after allocation (arrival counters) */
    int64_t ldraw, ldout;
    int32_t type, n_head, dim, vdim, col_q, col_g;
    float out_scale, eps;
} kf_rb_decay;
int kf_rb_decay_prefill(kf_ctx* ctx, const kf_rb_decay* a, const int32_t* meta, int n_rows, const int32_t* seqs, int n_seq, int max_n);
int kf_rb_decay_decode(kf_ctx* ctx, const kf_rb_decay* a, const int32_t* meta, int n_rows);
/* a layer's attention and its decayed sum of the same rows: kf_rb_attention_decode and kf_rb_decay_decode, in one launch where the rows are few */
int kf_rb_attention_decay_decode(kf_ctx* ctx, const kf_rb_attention* a, const kf_rb_decay* d, const int32_t* meta, int n_rows, int max_pos);
size_t kf_rb_decay_scratch(int type, int n_rows, int n_seq, int n_head, int dim, int vdim);

/* router: logits fp32 [n][ld] (+ bias [n_expert] in the batch's storage, may be NULL) -> the `top` largest of every row (ties: the lower expert) and the softmax over them;
 * rows whose meta position is < 0 (meta != NULL) choose nothing.  Then the pairs grouped by expert into the list.  experts: the arrays it points to are written. */
int kf_rb_route(kf_ctx* ctx, int type, const float* logits, int64_t ld, const void* bias, int n, const int32_t* meta, const kf_rb_experts* experts);
int kf_rb_list_tiles(int n, int top, int n_expert, int tile);

/* greedy pick over fp32 logits [n][ld], first maximum; row s advances slot s: d_tokens_out[s][pos] = id, d_state[s] = {id, pos + 1}.  Inactive rows (meta) are left
 * alone.  scratch: kf_rb_pick_scratch(n) bytes. */
int kf_rb_pick(kf_ctx* ctx, const float* logits, int64_t ld, int vocab, int n, const int32_t* meta, int32_t* d_state, int32_t* d_tokens_out, int tokens_stride, void* scratch);
size_t kf_rb_pick_scratch(int n);
/* fp32 logits row -> bf16 (what kf_sample reads) */
int kf_rb_to_bf16(kf_ctx* ctx, const float* src, kf_bf16* dst, size_t n);

#ifdef __cplusplus
}
#endif
#endif
