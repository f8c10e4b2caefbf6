/*
 * mlora_decoder.h - C ABI of the kernels for decoders with latent or tied attention, time mixing, experts and norms without
 * a weight per row.
 *
 * The library is built once per element type (libmlora_hip.so fp16, libmlora_bf16.so bfloat16, libmlora_f32.so fp32) with
 * the same entry points; "elements" below are of that type, and MLORA_F16 names it in dtype arguments.  The functions
 * declared here are in the bfloat16 and the fp32 library.  In the latter activations are row-major, weights are plain
 * [N, K] and fragment-ordered outputs are refused.  Conventions as in mlora.h.
 */
#ifndef MLORA_DECODER_H
#define MLORA_DECODER_H

#include "mlora.h"

#ifdef __cplusplus
extern "C" {
#endif

/* Residual stream x [T, Hp] fp32 (columns H..Hp-1 zero): x += the n_part blocks part[q][T][Hp], in order; with a branch
 * x += branch / rms(branch) * branch_w; then, where an output is given, out = x / rms(x) * gain (with `raw`: x itself), rms
 * over the H columns with eps inside the root; in fragment order and / or row-major [T, Hp]. */
int mlora_stream_norm(void* out_frag, void* out_row, float* x, const float* part, int n_part, const float* branch, const void* branch_w,
                      float eps, float gain, int raw, int T, int H, int Hp, void* stream);

/* Per-layer token input: out[t, n] = gelu_tanh(W[n] . x[t]) * table[ids[t], col0 + n] for n < dim, 0 for dim <= n < N.
 * mlora_token_gate takes x [T, K] and writes out in fragment order, W packed [N, K]; mlora_token_gate_mul takes the product
 * z [T, N] of a separate linear, row-major. */
int mlora_token_gate(void* out_frag, const void* xf, const void* Wp, const void* table, int ld_table, int col0, int dim, const int32_t* ids,
                     int V, int T, int K, int N, void* stream);
int mlora_token_gate_mul(void* out, const void* z, const void* table, int ld_table, int col0, int dim, const int32_t* ids, int V, int T, int N,
                         void* stream);

/* An elementwise norm dt(v) = tanh(alpha v) w + b; w == NULL: dt(v) = v.  w, b: elements [Hp], zero behind the width. */
typedef struct {
  const void* w;
  const void* b;
  float alpha;
} mlora_tanh_norm;

/* One step of the residual stream x [T, Hp] fp32:
 *   x_out = x + mult post(y + the n_part blocks part[q][T][Hp] + row_weight * the sum of the token's `top` rows)
 *   out   = pre(x_out), in fragment order (out_frag) and / or row-major with stride ld_row (out_row)
 * x NULL: zero; y and rows NULL: no branch (post and mult are not used); x_out may be x, or NULL.
 * With mu [5, Hp] the output is five mixes h + (h_prev - h) mu_s of h = pre(x_out), mix_stride elements apart; h_prev is the previous token's h
 * of the sequence: zero at position 0, shift [n_seq, Hp] (fp32, row tok_seq) for the sequence's first token of the pass, which also
 * stores the h of its last one (row tok_last[t]; NULL: itself) there.  A sequence's tokens are consecutive, and x_out is
 * not x then, unless there is no branch. */
typedef struct {
  float* x_out;
  const float* x;
  const float* y;
  const float* part;
  const void* rows;
  void* out_frag;
  void* out_row;
  const void* mu;
  float* shift;
  const int32_t* tok_seq;
  const int32_t* tok_pos;
  const int32_t* tok_last;
  mlora_tanh_norm post, pre;
  long mix_stride;
  int n_part, top, T, Hp, ld_row, n_seq;
  float mult, row_weight;
} mlora_stream_step_args;
int mlora_stream_step(const mlora_stream_step_args* args, void* stream);

/* y [T, N] fp32 = xf . Wp^T (bfloat16 library; fragment order, packed weight), K split over ks = mlora_gemv_ksplit(T, K, N) or fewer
 * slices: the reader of y adds the ks - 1 partial blocks part[q][T][N]. */
int mlora_linear_ksplit_store(float* y, float* part, int ks, const void* xf, const void* Wp, int T, int K, int N, void* stream);

/* y [T, N_main] = xf_g . Wp^T (bfloat16 library, T <= 64), row group g = row / group_rows (a multiple of 64) of the packed weight reading
 * the activation xf + g * x_stride; the N_ext rows behind N_main are a last group, whose result goes to y2
 * [mlora_gemv_groups_parts(K), T, N_ext] fp32 as partial sums over ranges of K. */
int mlora_gemv_groups_parts(int K);
int mlora_gemv_frag_groups(void* y, float* y2, const void* xf, long x_stride, int group_rows, const void* Wp, int T, int K, int N_main, int N_ext,
                           void* stream);
/* The same for more than 64 tokens, without the last group: mlora_narrow_linear, y [T, N] fp32 = xf . Wp^T for few rows N, takes that. */
int mlora_gemm_frag_groups(void* y, const void* xf, long x_stride, int group_rows, const void* Wp, int T, int K, int N, void* stream);
int mlora_narrow_linear(float* out, const void* xf, const void* Wp, int T, int K, int N, void* stream);

/* x [T, H] fp32 = table[ids[t]] * scale (zero for an id outside 0..V-1), and the same in elements (out_frag and / or out_row). */
int mlora_embed_scaled(float* x, void* out_frag, void* out_row, int ld_row, const void* table, const int32_t* ids, float scale, int T, int H, int V,
                       void* stream);

/* Time mixing (equations at the top of time_mix.hip): a recurrence per head over a matrix state, its decay, the norm of the
 * heads' outputs and their gate.  r, k, v, g [T, ld]; z [n_z, T, ld_z] fp32, R columns: partial sums of the
 * decay's low-rank projection (before the tanh); w2 [H * D, ld_w2], zero behind R; w0, u fp32 and norm,
 * each [H * D]; state [n_seq, H, D, D] fp32, updated.  segs [n_segs][4] int32 = {slot, first token, tokens, position of the first
 * token}; NULL: every token is a segment of its own (n_segs = T; a decode step).  y [T, ld_y], ld_y = H * D rounded up, zero behind H * D. */
int mlora_time_mix(void* y, int y_layout, int ld_y, const void* r, const void* k, const void* v, const void* g, int ld, const float* z, int n_z,
                   int ld_z, int R, const void* w2, int ld_w2, const float* w0, const float* u, const void* norm, float eps, float* state, int n_seq,
                   const int32_t* segs, int n_segs, const int32_t* tok_seq, const int32_t* tok_pos, int T, int H, int D, void* stream);

/* The same for prompts (bfloat16 library), in chunks on the matrix cores.  zp [T, 3, ld_zp]: tanh of the decay's low-rank projection as
 * the sum of three elements (mlora_tanh_parts: out [T, 3, N] from xf [T, K] and packed W [N, K]); w2 [H * D, ld_zp].  ranges [n_ranges][8]
 * int32 = {slot, first token, tokens, position of the first token, scratch state it starts from (-1: the slot's), scratch state that
 * takes what it adds (-1: none), whether it is its sequence's last, 0}: ranges of a sequence run side by side; a sequence of several
 * ranges has one scratch state per range and an entry in seqs [n_seqs][4] = {slot, position of its first token, first scratch state,
 * ranges}.  scratch: n_states * H * D * (D + 1) floats. */
int mlora_tanh_parts(void* out, const void* xf, const void* Wp, int T, int K, int N, void* stream);
int mlora_time_mix_prompt_served(int D);
int mlora_time_mix_prompt(void* y, int y_layout, int ld_y, const void* r, const void* k, const void* v, const void* g, int ld, const void* zp, int ld_zp,
                          const void* w2, const float* w0, const float* u, const void* norm, float eps, float* state, int n_seq,
                          const int32_t* ranges, int n_ranges, const int32_t* seqs, int n_seqs, float* scratch, size_t scratch_floats, int n_states,
                          int T, int H, int D, void* stream);

/* Latent attention (layouts at the top of latent_attention.hip).  mlora_latent_prep takes the token's projections qkv [T, ld]:
 * rotates the heads' query parts (columns off_rot .. + H rot) into the rows q + (t H + h) q_ld + q_off, padded to whole blocks of
 * 32, and, with c_norm, norms `gain` times the latent (off_c .. + R), rotates `gain` times the shared key part
 * (off_kr .. + rot) and stores both in the token's page slot.
 * With `lift` [H ceil32(R), lift_k] (packed; bfloat16 library) the same launch lifts the unrotated query parts - the first
 * lift_k columns per head of qkv - into columns 0 .. ceil32(R) of the rows (q_off = ceil32(R) then).
 * mlora_head_linear: y[t, h] = alpha W[h] . x[t, h].  mlora_latent_attn: causal softmax over the sequence's pages with scores
 * (q . cached) * scale, q [T, H, NB 32], and, with `sink`, exp(sink[h]) in the denominator; out [T, H, ceil32(R)].
 * splits > 1 needs a workspace.  mlora_latent_attn_out (splits > 1) takes the result through W_uv (packed [H vp, ceil32(R)]) in
 * the launch that merges the splits: y [T, H vp] in either layout. */
int mlora_latent_prep(void* q, int q_ld, int q_off, void* cache, const void* qkv, int ld, int off_rot, int off_c, int off_kr, float gain,
                      const void* c_norm, float eps, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                      const int32_t* tok_pos, const float* rope_cos, const float* rope_sin, int max_pos, int T, int H, int R, int rot,
                      int n_pages, int n_seq, const void* lift, int lift_k, void* stream);
int mlora_head_linear(void* y, int y_layout, long ldy, long head_y, const void* x, long ldx, long head_x, const void* W, int heads, int T,
                      int K, int N, float alpha, void* stream);
int mlora_latent_attn_splits(int T, int H, int max_ctx);
size_t mlora_latent_attn_workspace_bytes(int T, int H, int R, int splits);
int mlora_latent_attn(void* out, const void* q, const void* cache, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                      const int32_t* tok_pos, const float* sink, float scale, int T, int H, int R, int rot, int n_pages, int n_seq,
                      int splits, void* workspace, size_t workspace_bytes, void* stream);
int mlora_latent_attn_out(void* y, int y_layout, long ldy, const void* uv, int vp, const void* q, const void* cache, const int32_t* block_table,
                          int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos, const float* sink, float scale, int T, int H, int R,
                          int rot, int n_pages, int n_seq, int splits, void* workspace, size_t workspace_bytes, void* stream);

/* The same attention for prompts (bfloat16 library): makes the heads' keys and values of whole contexts in scratch memory and
 * attends over those.  phys [pages]: the cache pages of the contexts one after the other, each context padded with -1 to a
 * multiple of four pages; tiles [n_tiles][4] int32 = {first token, tokens (at most mlora_latent_prefill_tile_tokens), first
 * scratch page of its context, position of the first token}, one sequence each.  q [T, ld_q]: the heads' unrotated query parts, each
 * padded to 32 columns; q_rot [T, H, ceil32(rot)]; uk packed [H ceil32(dim), ceil32(R)], uv packed [H ceil32(vdim), ceil32(R)];
 * out [T, H ceil32(vdim)]. */
int mlora_latent_prefill_tile_tokens(void);
int mlora_latent_prefill_served(int dim, int rot, int vdim);
size_t mlora_latent_prefill_scratch_elems(int pages, int H, int dim, int rot, int vdim);
int mlora_latent_prefill(void* out, int out_layout, int ld_out, const void* q, int ld_q, const void* q_rot, const void* cache,
                         const int32_t* phys, int pages, const int32_t* tiles, int n_tiles, const void* uk, const void* uv, const float* sink,
                         float scale, int T, int H, int R, int dim, int rot, int vdim, int n_pages, void* scratch, size_t scratch_elems,
                         void* stream);

/* Tied attention (top of latent_attention.hip): H query heads in groups over G key/value heads of D columns, values = keys before
 * their norm.  mlora_tied_prep takes the projections y [T, ld] fp32 without biases (H query heads, then G key/value heads), adds the
 * biases, norms the queries (q_norm [D] is the queries' norm weight times the keys'), multiplies them with
 * 1 + temp_coef ln(floor((position + 1) / temp_every) + 1) (temp_every > 0) into q [T, H, ceil32(D)], and stores values and key scales in the
 * token's page slot.  mlora_tied_attn: causal softmax with scores (q . key) * scale - slopes[h] * distance, out [T, H ceil32(D)];
 * splits > 1 needs a workspace of mlora_latent_attn_workspace_bytes(T, H, D, splits).  mlora_tied_prefill (bfloat16 library): the same
 * for prompts over keys and values laid out in scratch memory; phys and tiles as for mlora_latent_prefill. */
int mlora_tied_prep(void* q, void* cache, float* key_scale, const float* y, int ld, const float* bias, const float* q_norm, float eps, float temp_coef,
                    float temp_every, const int32_t* block_table, int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos, int T, int H,
                    int G, int D, int n_pages, int n_seq, void* stream);
int mlora_tied_attn_splits(int T, int H, int G, int max_ctx);
int mlora_tied_attn(void* out, int out_layout, const void* q, const void* cache, const float* key_scale, const int32_t* block_table, int max_blocks,
                    const int32_t* tok_seq, const int32_t* tok_pos, const float* slopes, float scale, int T, int H, int G, int D, int n_pages,
                    int n_seq, int splits, void* workspace, size_t workspace_bytes, void* stream);
int mlora_tied_prefill_served(int D);
size_t mlora_tied_prefill_scratch_elems(int pages, int G, int D);
int mlora_tied_prefill(void* out, int out_layout, int ld_out, const void* q, const void* cache, const float* key_scale, const int32_t* phys, int pages,
                       const int32_t* tiles, int n_tiles, const float* slopes, float scale, int T, int H, int G, int D, int n_pages, void* scratch,
                       size_t scratch_elems, void* stream);

/* Mixture of experts.  mlora_moe_route: z = scale logits[t] + bias, the `top` largest per token (lower index on ties), softmax
 * over those.  mlora_moe_plan sorts the (token, choice) entries by expert into places - every
 * expert's start at a multiple of 16 - and tiles {expert, first place, places, 0} of mlora_moe_tile_rows places; perm holds
 * mlora_moe_max_places entries, tiles mlora_moe_max_tiles, n_tiles two numbers.  mlora_moe_linear multiplies tile by
 * tile with the experts' weights (one [N, K] block each): stage UP reads token rows x [T, K] and writes places, stage DOWN reads places
 * and writes entry rows [T top, N]; `act` is applied to alpha times the product.  Tiles of 256 places: the hidden places are in fragment
 * order, K % 64 == 0, and UP needs a workspace of places * K elements; else places are rows.  mlora_moe_combine: x[t] += the n_part blocks
 * part[q][T][N], then the sum over the choices of weight * row; out_frag (or NULL): the result in fragment order. */
#define MLORA_ACT_NONE  0
#define MLORA_ACT_RELU2 1   /* max(v, 0)^2 */
#define MLORA_ACT_GLU   2   /* up stage: silu(gate) * up, W a block of N gate rows and N up rows per expert (not in the fp32 library) */
#define MLORA_MOE_UP    0
#define MLORA_MOE_DOWN  1
int mlora_moe_route(int32_t* pick, float* weight, const float* logits, int ld, const float* bias, float scale, int T, int E, int top,
                    void* stream);
int mlora_moe_tile_rows(int T, int E, int top);
int mlora_moe_max_tiles(int T, int E, int top);
int mlora_moe_max_places(int T, int E, int top);
int mlora_moe_plan(int32_t* perm, int32_t* tiles, int32_t* n_tiles, const int32_t* pick, int T, int E, int top, void* stream);
/* mlora_moe_plan for `layers` layers whose experts are looked up by token id, table [layers, V, top]: perm, tiles and n_tiles layer
 * after layer. */
int mlora_moe_table_plan(int32_t* perm, int32_t* tiles, int32_t* n_tiles, const int32_t* table, const int32_t* ids, int layers, int V, int T, int E,
                         int top, void* stream);
int mlora_moe_linear(void* y, const void* x, const void* W, const int32_t* perm, const int32_t* tiles, const int32_t* n_tiles, int tile_rows,
                     int max_tiles, int places, int T, int K, int N, int top, int stage, int act, float alpha, void* workspace,
                     size_t workspace_elems, void* stream);
int mlora_moe_combine(float* x, const float* part, int n_part, const void* y, const float* weight, int T, int top, int N, void* out_frag,
                      void* stream);

#ifdef __cplusplus
}
#endif
#endif /* MLORA_DECODER_H */
