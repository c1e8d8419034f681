// k_layered.hpp — launchers of the layered-model kernels (k_layered.hip).  Host functions take
// a stream, never allocate or synchronise, and return 0 or an error with qie_last_error() text.
#pragma once

#include "qie_common.hpp"

namespace qie {
namespace lay {

// y[m, n] = sum_k A[m, k] W[n, k] (+ batch z: A + z sA, W + z sW, Y + z sY).  A fp32, rounded to
// bf16 on load when round_a; W fp32 or bf16 words; Y fp32.  grp_off (device, batch + 1 entries):
// batch z covers rows [grp_off[z], grp_off[z + 1]) of A and Y (M is then the largest row count a
// group can have).  Three kernels by shape: up to 32 rows a column-per-wave kernel, many rows of a
// bf16 model (mfma) MFMA tiles from memory, else 64 x 64 fp32 tiles through LDS; an element's sum
// never depends on what else the launch holds, only on which of the three ran.
struct LinearP {
    const float* A;
    int64_t lda;
    const void* W;
    int64_t ldw;
    float* Y;
    int64_t ldy;
    int M, N, K, batch;
    int64_t sA, sW, sY;
    int round_a;
    const int32_t* grp_off;
    int mfma;   // bf16 weights, many rows: the direct MFMA kernel may take the product (batched / grouped forms)
};
int linear(const LinearP& p, bool w_f32, hipStream_t st);

// Paged latent cache: page p at pool + p * page_stride elements; inside a page the rows of one
// caching layer start at layer_off and are D = R + rot wide: [c (R) | rotated shared key (rot)].
// Token t of slot s is row t % page_tokens of page table[s * max_pages + t / page_tokens].
struct LatentCache {
    void* pool;
    int64_t page_stride;
    const int32_t* table;
    int page_tokens, max_pages;
};

struct LatentPostP {
    float* proj;          // [T][ld]: q heads, then (own_kv) the compressed row and the shared key part
    int64_t ld;
    const int32_t* row_slot;
    const int32_t* row_pos;
    int heads, dim, rot, rot_dims, R, own_kv;
    const float* norm_w;  // [R]
    float eps;
    const float* rope_cos;   // [positions][rot_dims / 2]
    const float* rope_sin;
    LatentCache cache;
    int64_t layer_off;
    int interleaved;      // bf16 caches: also write the key-interleaved copy of c that follows the rows
    int rot_layout;       // 0: coordinate i turns with i + rot_dims / 2; 1: 2i with 2i + 1
    const float* kv;      // own_kv: where the compressed row and the shared key part are read from
    int64_t kv_ld;        //   ([T][kv_ld], columns 0 .. R + rot); null: the projection row after the q heads
};
int latent_post(const LatentPostP& p, bool cache_f32, int T, hipStream_t st);

struct LatentAttnP {
    const float* q_abs;   // [T][heads][R]
    const float* proj;    // rotated query parts are read from the projection rows
    int64_t ld;
    const int32_t* row_slot;
    const int32_t* row_pos;
    int heads, dim, rot, R, window;
    float scale;
    LatentCache cache;
    int64_t layer_off;
    float* out;           // [T][heads][R]
};
int latent_attention(const LatentAttnP& p, bool cache_f32, int T, hipStream_t st);

// The matrix-core form (k_latent_attn.hip; bf16 cache rows followed, per caching layer and page,
// by the key-interleaved copy of c: element ((t % page_tokens) / 4 * R + r) * 4 + t % 4).  A row
// group is up to 16 (token, head) rows of consecutive tokens of one slot: {first packed row,
// tokens, first head, heads per token}.  S splits over the keys; part_o [groups * S][16][R] and
// part_ml [groups * S][16][2] are scratch.
struct LatentAttnMfmaP {
    const float* q_abs;
    const float* proj;
    int64_t ld;
    const int32_t* row_slot;
    const int32_t* row_pos;
    const int4* groups;
    int n_groups, S;
    int heads, dim, rot, R, window;
    float scale;
    LatentCache cache;
    int64_t layer_off;
    float* part_o;
    float* part_ml;
    float* out;           // [T][heads][R]
};
// Row groups a wave takes together: the group list of a step holds, per entry, a multiple of
// kLatentQG groups (padded with empty groups {row, 0, 0, 1}), and consecutive groups of a unit
// belong to one slot.
constexpr int kLatentQG = 1;   // 2 measured slower at kv_rank 256 (one wave per SIMD), and spills at 512
bool latent_attention_mfma_fits(int R, int rot);
int latent_attention_mfma(const LatentAttnMfmaP& p, hipStream_t st);

// ------------------------------------------------------------------ grouped-query attention
// (k_mixers.hip)  Paged K / V rows: inside a page the K rows of one cache region start at k_off
// and are kv_heads * dim wide, its V rows at v_off, kv_heads * vdim wide (LatentCache names the
// pool, its block table and the page geometry).
//
// gqa_post: per row of the fused projection, every query and key head is RMS-normed over dim
// (qk_norm: 0 no, 1 with the weight qn_w / kn_w, 2 without one; 3: all query heads of the row are normed as one vector
// with weights qn_w [heads * dim], all key heads as another with kn_w [kv_heads * dim]), its first rot_dims coordinates
// are turned by the row's position (layout 0: i with i + rot_dims / 2; 1: 2i with 2i + 1); queries
// go back in place, keys to the cache.  Values: v_col < 0 caches the key as projected (before its
// norm) as the value; else W_v's columns, turned over all vdim coordinates when rot_values.
struct GqaPostP {
    float* proj;
    int64_t ld;
    int q_col, k_col, v_col;
    const int32_t* row_slot;
    const int32_t* row_pos;
    int heads, kv_heads, dim, vdim;
    int qk_norm;
    const float* qn_w;
    const float* kn_w;
    float eps;
    int rot_dims, rot_layout;
    const float* rope_cos;    // [positions][rot_dims / 2]
    const float* rope_sin;
    int rot_values;
    const float* vrope_cos;   // [positions][vdim / 2]
    const float* vrope_sin;
    LatentCache cache;
    int64_t k_off, v_off;
    int v_transposed;         // V rows of a page stored [kv_heads][vdim][page_tokens]
    // q_temp_every > 0: the normed query is multiplied by 1 + q_temp_coef * ln((pos + 1) / every + 1),
    // the division rounded down
    int q_temp_every;
    float q_temp_coef;
    const float* q_bias;      // [heads * dim] / [kv_heads * dim] or null: added to q / k as they leave the projection
    const float* k_bias;      //   (a key cached as the value carries its bias)
    const float* v_bias;      // [kv_heads * vdim] or null: added to v as it leaves the projection
    // optional: the step's groups of up to 16 consecutive rows {first packed row, rows, slot, first position};
    // transposed values of prompt-sized steps are then written 16 tokens at a time
    const int4* groups;
    int n_groups;
    int q_only;               // the layer reads another layer's keys and values: no key or value columns, nothing cached
};
int gqa_post(const GqaPostP& p, bool cache_f32, int T, hipStream_t st);

// Softmax attention of every (row, head) over the keys its mask lets it see (mask 0: all j <= i;
// 1: the last mask_size and, of the earlier ones, the first mask_keep of the sequence; 2: those with
// j / mask_size == i / mask_size); score = q.k * scale
// (soft-capped when softcap > 0) - r1[h] * ln(1 + r2[h] * (i - j)) when r1 is set.  rot_values: the weighted sum is turned back
// by the row's position.  The result times out_scale goes to out[t * ld_out + out_col + h * vdim
// ...] (and its bf16 image).
struct GqaAttnP {
    const float* proj;
    int64_t ld;
    int q_col;
    const int32_t* row_slot;
    const int32_t* row_pos;
    int heads, kv_heads, dim, vdim;
    int mask, mask_size;
    float scale;
    const float* r1;
    const float* r2;
    int rot_values, rot_layout;
    const float* vrope_cos;
    const float* vrope_sin;
    LatentCache cache;
    int64_t k_off, v_off;
    int v_transposed;
    float out_scale;
    float* out;               // null: only the bf16 image is wanted
    uint16_t* out_bf;
    int64_t ld_out;
    int out_col;
    const float* slopes;      // [heads] or null: the score also loses slopes[h] * (i - j)
    const float* pb;          // [heads] or null; set: a visible key's weight is sigmoid(score + pb[h]),
                              // and the weights of a row are used as they are (no softmax)
    int gate_col;             // >= 0: head h's result times sigmoid(proj[t * ld + gate_col + h])
    int gate_elem;            // with gate_col: one gate per coordinate, proj[t * ld + gate_col + h * vdim + c]
    const float* sink;        // [heads] or null: exp(sink[h]) joins the softmax denominator (no key, no value)
    int mask_keep;            // mask 1 only, else 0
    float softcap;            // > 0: the scaled score s becomes softcap * tanh(s / softcap) before biases
};
int gqa_attention(const GqaAttnP& p, bool cache_f32, int T, hipStream_t st);
// The matrix-core form for bf16 caches whose V rows are stored transposed (v_transposed: inside a
// page [kv_heads][vdim][page_tokens], so that 4 keys of one value coordinate are one 8-byte load;
// page_tokens a multiple of 32), dim and vdim 32, 64, 96, 128, 192 or 256.  A wave takes
// up to 16 (token, head) columns of one slot that share a key head: 16 consecutive tokens of one
// head, or - for groups of few tokens, see pack - the heads of one key head per token.  groups: {first
// packed row, tokens (<= 16), slot, first position}.  S > 1 splits every wave's keys S ways
// (decoding: few columns, many keys); the partial sums meet in a second pass.  part_o
// [groups * tiles * S][16][vdim], part_ml [...][16][2] floats of scratch (tiles = 4 * ceil(heads / 4)).
struct GqaAttnMfmaP {
    GqaAttnP a;
    const int4* groups;
    int n_groups, S;
    float* part_o;
    float* part_ml;
    // 1: groups of few tokens pack the heads of a key head into a wave's columns, every wave loads
    // its own fragments (head ratios that are no multiple of 4); 0: one head per wave, the four
    // waves of a workgroup share their key head's tiles through LDS (ratios that are)
    int pack;
};
bool gqa_attention_mfma_fits(int dim, int vdim, int page_tokens);
int gqa_attention_mfma(const GqaAttnMfmaP& p, hipStream_t st);

// ------------------------------------------------------------------ gated linear recurrence
// Per entry {first packed row, rows, slot, first position} and head: S [dim][vdim] (fp32, at
// state + slot * slot_stride + state_off) runs through the entry's rows in order,
// S = diag(f) S + (1 - f) v^T, o = S^T q, with q = silu(proj[q_col ...]),
// f = lower + (1 - lower) * sigmoid(proj[f_col ...] + f_bias); an entry whose first position is 0
// starts from S = 0.  Raw o -> out [T][heads * vdim].
struct GatedScanP {
    const float* proj;
    int64_t ld;
    int q_col, f_col, v_col;
    const int4* entries;
    int n_entries;
    int heads, dim, vdim;
    const float* f_bias;
    const float* lower;
    float* state;
    int64_t slot_stride, state_off;
    float* out;
    // mode 0: the recurrence itself (state read unless the entry starts at position 0, advanced,
    // written back); decay (optional) receives the product of the entry's gates, [entries][heads][dim].
    // mode 1: the state is only read, every row's q is scaled by the product of the gates from the
    // entry's first row to this row, and out receives S^T q: the share of an incoming state in the
    // outputs of rows that were scanned from a zero state (the caller adds the two).
    int mode;
    float* decay;
};
int gated_scan(const GatedScanP& p, hipStream_t st);
// Long entries in pieces: `chunks` lists pieces {first packed row, rows, piece index, 0} in entry
// order, `spans` one {first piece, pieces, slot, first position} per entry.  gated_scan (mode 0)
// over the pieces from zero states gives piece-local outputs, end states s_loc [pieces][heads *
// dim * vdim] and gate products; gated_carry walks an entry's pieces in order (s_in[c] = state
// entering piece c, starting from the slot's state or zero; the slot's state = what leaves the
// last piece); gated_scan (mode 1) over the pieces with s_in gives the incoming states' share.
// Same sums as the row-by-row recurrence up to fp32 rounding.
struct GatedCarryP {
    const int4* spans;
    int n_spans;
    int heads, dim, vdim;
    const float* s_loc;
    const float* decay;
    float* s_in;
    float* state;
    int64_t slot_stride, state_off;
};
int gated_carry(const GatedCarryP& p, hipStream_t st);
// ------------------------------------------------------------------ minGRU
// Per entry {first packed row, rows, index, first position} and channel c < n: with
// z = sigmoid(proj[z_col + c] + z_b[c]), u = proj[x_col + c] + x_b[c], cand = u >= 0 ? u + 1/2 :
// sigmoid(u), the state runs through the entry's rows in order, S = (1 - z) S + z cand, and
// out[row, c] = S * silu(proj[g_col + c]) (with its bf16 image).  fp32 throughout.
// init: the state an entry starts from, at init + index * init_stride (+ init_off); null, or (when
// init_if_pos) an entry whose first position is 0: zero.  end / decay (optional, same addressing
// with end_stride): the state after the entry's last row, the product of its (1 - z).  out may be
// null (a pass that only wants end and decay).
struct MinGruScanP {
    const float* proj;
    int64_t ld;
    int z_col, x_col, g_col;
    const float* z_b;
    const float* x_b;
    const int4* entries;
    int n_entries, n;
    const float* init;
    int64_t init_stride, init_off;
    int init_if_pos;
    float* end;
    float* decay;
    int64_t end_stride, end_off;
    float* out;
    uint16_t* out_bf;
    int64_t ld_out;
};
int mingru_scan(const MinGruScanP& p, hipStream_t st);
// Long entries in pieces (lists as for gated_carry): s_in[c] = the state entering piece c, from the
// slot's state (or zero at position 0) through S <- decay[c] S + s_loc[c]; the slot's state = what
// leaves the entry's last piece.
struct MinGruCarryP {
    const int4* spans;
    int n_spans, n;
    const float* s_loc;
    const float* decay;
    float* s_in;
    float* state;
    int64_t slot_stride, state_off;
};
int mingru_carry(const MinGruCarryP& p, hipStream_t st);

// out[t, out_col + h * vdim + c] = scale * o[t, h, c] / sqrt(mean_c o^2 + eps) * w[c], o = o1 + o2 when o2
// gate (optional): the result is also multiplied by sigmoid(gate[t * ld_gate + h * vdim + c]), or silu of it
// (gate_silu); ld_gate 0: heads * vdim
int head_norm_rows(const float* o, const float* o2, const float* w, float eps, float scale, int heads, int vdim, int T, float* out,
                   uint16_t* out_bf, int64_t ld_out, int out_col, hipStream_t st, const float* gate = nullptr, int64_t ld_gate = 0,
                   int gate_silu = 0);
// out[t, c] = y[t, c] * silu(z[t * ld_z + c]), then every one of `parts` equal parts of the n columns divided by its
// root mean square and multiplied by w[c] (with its bf16 image)
int gated_norm_parts(const float* y, const float* z, int64_t ld_z, const float* w, float eps, int n, int parts, int T, float* out,
                     uint16_t* out_bf, int64_t ld_out, hipStream_t st);
// Rows of W, two norms of one row: x = xin + v (when v) + v2 (when v2) + v3 (when v3) + add (when add); h1 = rms(x) w1, h2 = rms(x) w2
// (each fp32, as its bf16 image, or both; null w1: neither norm is made, null w2: only the first)
struct NormPairP {
    float* x;
    const float *xin, *v, *v2, *add;
    const float *w1, *w2;
    float *h1, *h2;
    uint16_t *h1_bf, *h2_bf;
    int T, W;
    float eps;
    const float* v3;
    // both set (then v and v2 are too): v and v2 are RMS-normed with these weights and scaled before they are added
    const float *v_w, *v2_w;
    float v_scale, v2_scale;
};
int norm_pair(const NormPairP& p, hipStream_t st);
// (head_norm_rows, gated_norm_parts, silu_mul: with a null fp32 output only the bf16 image is written)

// ------------------------------------------------------------------ residual streams (k_streams.hip)
// n residual rows per token, X + s * plane (rows of W).  With y (a sublayer's result, [T][W]) the rows
// are replaced, all at once from the old ones, by x_t = sum_s mix[s * n + t] x_s + out[t] y.  With `in`
// the read-out u = sum_s in[s] x_s of the (new) rows is normed, h = u / sqrt(mean(u^2) + eps) *
// (w_one + wn), with its bf16 image.  sum (optional) receives the plain sum of the (new) rows.
struct StreamStepP {
    float* X;
    int64_t plane;
    int n;
    const float* y;
    const float* mix;
    const float* out;
    const float* in;
    const float* wn;
    float w_one, eps;
    float* h;
    uint16_t* h_bf;
    float* sum;
    int T, W;
};
int stream_step(const StreamStepP& p, hipStream_t st);

// Causal convolution over time per channel on the packed rows of a step: out[t, c] = (bias ? bias[c] : 0) +
// (residual ? in[t, c] : 0) + sum_j w[c * taps + j] in[t - (taps - 1 - j), c], then silu when asked.
// Rows before an entry's first come from the slot's state ([taps - 1][C] floats at state + slot *
// slot_stride + state_off: the inputs at the taps - 1 positions before the entry, oldest first), rows
// before position 0 are zero.  row_k: a row's index inside its entry.  causal_conv_state moves the
// state on by the step's entries {first packed row, rows, slot, first position}; run it after
// causal_conv (which reads the old state) and before `in` is overwritten.
struct CausalConvP {
    const float* in;
    int64_t ld_in;
    int col, C, taps;
    const float* w;
    const int32_t* row_slot;
    const int32_t* row_pos;
    const int32_t* row_k;
    float* state;
    int64_t slot_stride, state_off;
    int residual, silu;
    float* out;
    int64_t ld_out;
    uint16_t* out_bf;
    const int4* entries;
    int n_entries;
    const float* bias;    // [C] or null
    const float* in_bias; // [C] or null: added to every input of the sequence (`in` and the state hold inputs without it)
};
int causal_conv(const CausalConvP& p, int T, hipStream_t st);
int causal_conv_state(const CausalConvP& p, hipStream_t st);
// Both in order; steps of at most kConvFusedRows rows in one launch (a thread per entry and channel)
constexpr int kConvFusedRows = 64;
int causal_conv_advance(const CausalConvP& p, int T, hipStream_t st);
// out[t, c] = in[t, col + c] / sqrt(mean_c in^2 + eps) * (w_one + w[c]), c < n (out may be in + col)
int rms_rows(const float* in, int64_t ld_in, int col, int n, const float* w, float w_one, float eps, float* out, int64_t ld_out,
             uint16_t* out_bf, int T, hipStream_t st);

// ------------------------------------------------------------------ gated delta rule (k_delta.hip)
// qkv [T][ld_qkv]: q (G heads of dim), k (G x dim), v (H x vdim) after their convolutions.  delta_prep,
// in place: q and k heads to unit length (x / sqrt(sum x^2 + 1e-6)), q also times dim^(-1/2);
// proj[t, b_col + h] = sigmoid of itself; a [T][H * dim] = exp(-exp_a[h] * softplus(a + dt_bias)).
// a null: one decay per head, proj[t, a_col + h] = exp(-exp_a[h] * softplus(itself + dt_bias[h])).
struct DeltaPrepP {
    float* qkv;
    int64_t ld_qkv;
    float* proj;
    int64_t ld;
    int b_col;
    float* a;
    const float* dt_bias;   // [H * dim]
    const float* exp_a;     // [H]: exp(A_log)
    int H, G, dim, vdim;
    int a_col;
};
int delta_prep(const DeltaPrepP& p, int T, hipStream_t st);
// Per entry {first packed row, rows, slot, first position} and head h (key head h / (H / G)), the fp32
// state S [dim][vdim] at state + slot * slot_stride + state_off + h * dim * vdim walks the rows in
// order: S = diag(g) S; u = beta (v - S^T k); S += k u^T; out[t, h] = S^T q.  An entry whose first
// position is 0 (or read_state = 0) starts from S = 0; write_state = 0 leaves the slot's state alone.
struct DeltaScanP {
    const float* qkv;
    int64_t ld_qkv;
    const float* beta;      // beta[t * ld_beta + h]
    int64_t ld_beta;
    const float* g;         // [T][H * dim]; with ld_g > 0 one decay per head: g[t * ld_g + h]
    int64_t ld_g;
    const int4* entries;
    int n_entries;
    int H, G, dim, vdim;
    float* state;
    int64_t slot_stride, state_off;
    int read_state;         // 0: start from zero; 1: read the state unless the entry starts at position 0; 2: always read
    int write_state;
    float* out;             // [T][H * vdim]
    // pieces of long entries (entries {first packed row, rows, piece index, 0}, state = per-piece end states): with
    // trans [pieces][H][dim][dim] the piece's transition matrix M (s_end = M s_in + s_loc) is written there and
    // w_out [T][H * dim] receives w_t = M_t^T q_t, M_t the transition from the piece's start to row t
    float* trans;
    float* w_out;
};
int delta_scan(const DeltaScanP& p, hipStream_t st);
// Walks every entry's pieces (spans {first piece, pieces, slot, first position}): s_in[c] = the state entering piece
// c, from the slot's state (zero at position 0) through s <- M_c s + s_loc[c]; the slot's state = what leaves the
// last piece (write_state).  s_loc, s_in [pieces][H][dim][vdim].
struct DeltaCarryP {
    const int4* spans;
    int n_spans;
    int H, dim, vdim;
    const float* s_loc;
    const float* trans;
    float* s_in;
    float* state;
    int64_t slot_stride, state_off;
    int write_state;
};
int delta_carry(const DeltaCarryP& p, hipStream_t st);
// out[t, h, :] += s_in[piece of t][h]^T w[t, h, :] over the pieces {first packed row, rows (<= max_rows), piece index, 0}
struct DeltaApplyP {
    const int4* chunks;
    int n_chunks, max_rows;
    int H, dim, vdim;
    const float* s_in;
    const float* w;
    float* out;
};
int delta_apply(const DeltaApplyP& p, hipStream_t st);
// ------------------------------------------------------------------ decayed linear recurrences (k_linrec.hip)
// Per entry {first packed row, rows, slot (or piece), first position} and head h, the fp32 state S [dim][vdim] at
// state + index * stride + off + h * dim * vdim walks the rows in order:
//   S = diag(a) S + m k v^T,  o = q_scale S^T q (+ skip[h] v)  ->  out[t * heads * vdim + h * vdim + c]
// q(t, h) = q + t ldq + (h / rep) dim, k alike (rep heads share a q / k row), v(t, h) = v + t ldv + h vdim.
// log_decay set: a = exp(log_decay[t * heads * dim + h dim + d]), m = 1.  dt set: one decay per head,
// dt_h = softplus(dt[t ld_dt + h] + dt_bias[h]), a = exp(-a_h[h] dt_h), m = dt_h.
// An entry whose first position is 0 starts from S = 0 (init_if_pos), else from the state at init.
struct LinRecP {
    const float *q, *k, *v;
    int64_t ldq, ldk, ldv;
    int rep;
    float q_scale;
    const float* log_decay;
    const float* dt;
    int64_t ld_dt;
    const float *dt_bias, *a_h, *skip;
    // linrec_step alone: the log decays straight from their low-rank projection (as low_rank_log_sigmoid makes them)
    const float* lr_in;
    int64_t ld_lr;
    const void* lr_w;
    int lr_w_f32, rank;
    const float* lr_bias;
    float inv_tau;
    int heads, dim, vdim;
    const int4* entries;
    int n_entries;
    const float* init;        // null: every entry starts from zero
    int64_t init_stride, init_off;
    int init_if_pos;
    float* end;               // null: the state after the last row is not kept
    int64_t end_stride, end_off;
    float* decay;             // optional [entries][heads * dim]: the product of the entry's decays
    float* out;               // null: only end and decay are wanted
};
// Rows in order on the vector units: entries of few rows (any dim up to 512)
int linrec_step(const LinRecP& p, hipStream_t st);
// 16 rows at a time on the fp32 matrix cores, the state in registers (dim up to 256)
bool linrec_walk_fits(int dim, int vdim);
int linrec_walk(const LinRecP& p, hipStream_t st);
// Walks every entry's pieces (spans {first piece, pieces, slot, first position}): s_in[c] = the state entering piece
// c, from the slot's state (zero at position 0) through s <- decay[c] s + s_loc[c]; the slot's state = what leaves
// the last piece.
struct LinRecCarryP {
    const int4* spans;
    int n_spans;
    int heads, dim, vdim;
    const float *s_loc, *decay;
    float* s_in;
    float* state;
    int64_t slot_stride, state_off;
};
int linrec_carry(const LinRecCarryP& p, hipStream_t st);
// ------------------------------------------------------------------ real-gated linear recurrent unit (k_rglru.hip)
// u [T][ld_u]: the convolved input, n = blocks * bs channels.  Gates of channel c of block b: r = sigmoid(R_b[c] . u_b +
// r_b[c]), i likewise; log a = -decay[c] * r, S_t = a S_(t-1) + sqrt(1 - a^2) i u.  w: [blocks][2 bs][bs], a block's R rows
// then its I rows, bf16 words or fp32 (w_f32).  All products and sums are fp32 (bf16 weights enter exactly, u as the sum
// of three bf16 parts that hold its 24 bits).
struct RgLruP {
    const float* u;
    int64_t ld_u;
    const void* w;
    int w_f32;
    const float *r_b, *i_b, *decay;   // [n]; decay = the design's constant * softplus(lam)
    int blocks, bs;
    float *a, *b;                     // [T][n]: a and sqrt(1 - a^2) i u (rglru_gates writes them, rglru_scan reads them)
    float* z;                         // rglru_gates: scratch [T][2 n] where the matrix-core form does not take the shape
    // the recurrence
    const float* y;                   // [T][ld_y]: the other branch before its bias and gelu
    int64_t ld_y;
    const float* y_b;                 // [n]
    const int32_t *row_slot, *row_pos, *row_k;
    const int4* entries;              // as in MinGruScanP
    int n_entries;
    const float* init;
    int64_t init_stride, init_off;
    int init_if_pos;
    float *end, *decay_out;
    int64_t end_stride, end_off;
    float* out;                       // [T][ld_out] S * gelu_tanh(y + y_b); null: only the bf16 image
    uint16_t* out_bf;
    int64_t ld_out;
    int want_out;                     // 0: only end and decay_out
};
int rglru_gates(const RgLruP& p, int T, hipStream_t st);
bool rglru_gates_mfma_fits(int bs, bool w_f32);
int rglru_scan(const RgLruP& p, hipStream_t st);
// Steps of few rows: gates and recurrence in one launch (state at init = end), a wave per channel, a lane per row.
// chain: no entry has more rows
constexpr int kRgLruStepRows = 64;
int rglru_step(const RgLruP& p, int T, int chain, hipStream_t st);

// out[t, c] = log(sigmoid(z)) / tau, z = sum_r w[c * rank + r] in[t * ld_in + r] + bias[c]; c < n
int low_rank_log_sigmoid(const float* in, int64_t ld_in, int rank, const void* w, bool w_f32, const float* bias, float tau, int n, int T,
                         float* out, hipStream_t st);

// Rows of W: x = xin + (wb ? rms(v) * (w_one + wb) : v) (when v) + add (when add); then (when wn)
// h = rms(x) * (w_one + wn) with its bf16 image.  xin may be x.  w_one = 1: weight vectors stored
// around zero; 0: plain weights.
// copies > 1: h is written `copies` times, `plane` elements apart (the rows of several residual streams start equal).
int add_norm(float* x, const float* xin, const float* v, const float* wb, const float* add, const float* wn, float* h, uint16_t* h_bf,
             int T, int W, float eps, hipStream_t st, float w_one = 1.0f, int copies = 1, int64_t plane = 0);

// The producers below also write the bf16 image of their result when the *_bf pointer is set
// (bf16 engines: the next product reads it; no separate rounding pass).
// out[t] = E[tok[t]] * scale; with pos (the rows' positions) and freq (double [ceil(W / 2)]) the
// sinusoidal position vector is added: entry 2i = sin(pos * freq[i]), entry 2i + 1 = cos of it
int embed_rows(const void* E, bool w_f32, const int32_t* tok, float* out, uint16_t* out_bf, int T, int W, int vocab,
               hipStream_t st, float scale = 1.0f, const int32_t* pos = nullptr, const double* freq = nullptr);
int head_gate(float* v, uint16_t* v_bf, const float* proj, int64_t ld, int g_col, int heads, int vd, int T, hipStream_t st);
// y = (x ? x : 0) + gain * v / sqrt(mean(v^2) + eps), rows of W
int postnorm_add(const float* x, const float* v, float* y, uint16_t* y_bf, int T, int W, float gain, float eps, hipStream_t st);
// out[i] = gain * rms(x[rows[i]]) (* (w_one + w1p) when w1p)
int final_rows(const float* x, const int32_t* rows, float* out, uint16_t* out_bf, int n, int W, float gain, const float* w1p,
               float eps, hipStream_t st, float w_one = 1.0f);
int depth_mix(const float* stack, int64_t stride, const float* a, int n, float* x, uint16_t* x_bf, int64_t count, hipStream_t st);
// a[m * ld_a + j] = act(gu[m, j]) * gu[m, ff + j]; act 0: silu, 1: the tanh form of gelu, 2: g sigmoid(1.702 g) (u + 1)
// with g = min(gu[m, j], limit), u = gu[m, ff + j] clamped to +-limit, 3: relu; ld_a 0: ff; ld_gu (rows of gu) 0: 2 ff
int silu_mul(const float* gu, float* a, uint16_t* a_bf, int64_t M, int ff, hipStream_t st, int act = 0, float limit = 0.f,
             int64_t ld_a = 0, int64_t ld_gu = 0);
// x = c tanh(x / c) in place, n elements
int softcap(float* x, int64_t n, float c, hipStream_t st);
// a = ap u^2 + u / 2 where u > 0, else aq (exp(u) - 1 - u) + u / 2; n elements
int xielu(const float* u, float* a, uint16_t* a_bf, int64_t n, float ap, float aq, hipStream_t st);
// mode 0: score = sigmoid(z) of the `top` largest z = W_r y; mode 1: z = W_r y + bias, score = the
// softmax over the `top` largest z alone.  Ties: the lower index.
int route_topk(const float* y, const void* Wr, const float* bias, bool w_f32, int T, int W, int E, int top, int mode, int32_t* sel,
               float* score, hipStream_t st);
// s = softmax over all E router outputs; chosen by s + corr inside the `keep` best of `groups` equal
// groups of neighbours (a group ranks by its largest s + corr), `top` of them; score = s of the
// chosen / (their sum + 1e-20) * scale.  Ties: the lower index.
int route_grouped(const float* y, const void* Wr, const float* corr, bool w_f32, int T, int W, int E, int top, int groups, int keep,
                  float scale, int32_t* sel, float* score, hipStream_t st);
int moe_group(const int32_t* sel, int n, int E, int32_t* cnt, int32_t* off, int32_t* slot_of, hipStream_t st);
// score (may be null: 1) scales the gathered input rows / the combined output rows
int moe_gather(const float* y, const float* score, const int32_t* slot_of, int T, int top, int W, float* xg, uint16_t* xg_bf,
               hipStream_t st);
// sel / n_real / y: a chosen expert >= n_real is an identity expert whose output is the row's input y
int moe_combine(const float* yd, const int32_t* slot_of, const float* score, int T, int top, int W, float* f, hipStream_t st,
                const int32_t* sel = nullptr, int n_real = 0, const float* y = nullptr);
int argmax_rows(const float* x, int M, int64_t V, int32_t* ids, hipStream_t st);
int rows_to_bf16(const float* x, uint16_t* y, int64_t n, hipStream_t st);
int rows_to_bf16_strided(const float* x, int64_t ldx, uint16_t* y, int64_t ldy, int64_t M, int K, hipStream_t st);
int bf16_to_f32(const uint16_t* x, float* y, int64_t n, hipStream_t st);

}  // namespace lay
}  // namespace qie
