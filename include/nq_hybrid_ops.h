/* C ABI of libnq_hybrid.so: the kernels of decoders that a configuration describes layer by layer -- sandwich norms on
 * an fp32 residual stream, attention with whole-projection q/k norm, interleaved rotary, a chunked or sliding-window mask
 * and sinks over the paged KV cache, gated linear attention with an fp32 recurrent state, mixtures of experts with an input-side weight,
 * latent attention, selective scans with a short convolution, residuals of several streams (hyper-connections), dense
 * skinny products, and the bookkeeping of a decode step.
 *
 * Conventions: device pointers, dense row-major tensors unless a row stride is given, `dtype` is NQH_BF16 or NQH_F32
 * for every activation and weight of a call, `stream` is a hipStream_t as void*.  The return value is 0 or an NQH_ERR
 * code, nqh_last_error() holds the message of the calling thread's last failure.  All arithmetic is fp32; matrix
 * products in bf16 accumulate in fp32.  The reference has no model of this kind: these entries have no counterpart. */
#ifndef NQ_HYBRID_OPS_H_
#define NQ_HYBRID_OPS_H_

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum nqh_dtype { NQH_BF16 = 1, NQH_F32 = 2 };
enum nqh_status { NQH_OK = 0, NQH_ERR_ARG = 1, NQH_ERR_UNSUPPORTED = 2, NQH_ERR_WORKSPACE = 3, NQH_ERR_HIP = 4 };

/* What follows a matrix product: nothing, the square of max(v, 0), or param * tanh(v / param). */
enum nqh_activation { NQH_ACT_NONE = 0, NQH_ACT_RELU2 = 1, NQH_ACT_SOFTCAP = 2 };

const char* nqh_last_error(void);

/* The step between two sublayers, on the fp32 residual stream x [rows, width]:
 *   x  = 0 if init else x
 *   x += RMSNorm(sum of the `y_parts` rows of y [rows, y_parts, width]) * post_weight     (y may be NULL)
 *   x += table[ids[r]]                                                                   (ids may be NULL)
 *   h  = RMSNorm(x) * next_weight                                                        (h may be NULL)
 * post_weight NULL adds the sum of the parts as it is.  RMSNorm(v) = v / sqrt(mean(v^2) + eps).  width <= 8192. */
int nqh_residual_norm(float* x, int init, const void* y, int64_t y_parts, const void* post_weight, const int64_t* ids,
                      const void* table, int64_t table_rows, const void* next_weight, void* h, int64_t rows,
                      int64_t width, float eps, int dtype, void* stream);

/* The step between two sublayers with hyper-connections, on the fp32 residual x [rows, streams, width]:
 *   x[., s]  = table[ids[r]] for every stream s                              (ids given: the start; y must be NULL)
 *   x[., t]  = sum_s mix[s, t] x[., s] + w_out[t] y, all at once             (y [rows, width] may be NULL)
 *   h        = RMSNorm(sum_s w_in[s] x[., s]) * norm_weight                  (h may be NULL; w_in NULL: ones)
 * mix [streams, streams], w_out and w_in [streams] have the call's dtype.  width <= 8192, streams <=
 * nqh_hyper_max_streams. */
int64_t nqh_hyper_max_streams(void);
int nqh_hyper_norm(float* x, const int64_t* ids, const void* table, int64_t table_rows, const void* y, const void* mix,
                   const void* w_out, const void* w_in, const void* norm_weight, void* h, int64_t rows, int64_t streams,
                   int64_t width, float eps, int dtype, void* stream);

/* x [count] = activation(x), in place; act is an nqh_activation. */
int nqh_activate(void* x, int64_t count, int act, float param, int dtype, void* stream);

/* nqh_residual_norm with the router and the plan of the layer behind it in the same launch, for few rows (see
 * nqh_residual_norm_route_supported): h as above (required), expert / weight as nqh_router_topk on h, order / tiles as
 * nqh_moe_plan.  `counter`: one int32 that is zero before the call and after it. */
int nqh_residual_norm_route_supported(int64_t rows, int64_t width, int64_t experts);
int nqh_residual_norm_route(float* x, int init, const void* y, int64_t y_parts, const void* post_weight,
                            const int64_t* ids, const void* table, int64_t table_rows, const void* next_weight, void* h,
                            const void* router, int32_t* expert, float* weight, int32_t* order, int32_t* tiles,
                            int32_t* counter, int64_t rows, int64_t width, int64_t experts, int64_t top,
                            int64_t tile_rows, int64_t max_tiles, float eps, int dtype, void* stream);

/* qkv [rows, heads * dim + kv_heads * (dim + vdim)]: q and k are RMS-normalised over the whole projection (weights of
 * that size; NULL: no norm) and rotated, pairs (2i, 2i + 1) of the first rot_dims dims of every head by the angle whose
 * cosine and sine (any magnitude factor included) are cos_sin [max_positions, rot_dims] = cos | sin at positions[row].
 * q goes to q_out [rows, heads, k_row]; k and v to their cache rows [block][kv_head][token][k_row | v_row] at slot
 * slots[row] = block * block_size + offset (outside [0, num_slots): not written).  Only the first dim (vdim) elements
 * of a padded row are written; q_out padding is zeroed.  dim and rot_dims even. */
int nqh_qk_norm_rope_store(const void* qkv, const void* q_weight, const void* k_weight, const float* cos_sin,
                           const int64_t* positions, const int64_t* slots, void* q_out, void* k_cache, void* v_cache,
                           int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t rot_dims,
                           int64_t k_row, int64_t v_row, int64_t max_positions, int64_t num_slots, int64_t block_size,
                           float eps, int dtype, void* stream);

/* Attention of the query tokens of a prompt pass over their sequences' cached keys (their own included).  The pass is a
 * list of segments, int32 [.][3] = first row in q, rows, position of the first row in its sequence; segment s has the block
 * table block_tables[s] (int32 [.][max_blocks]).  A query at position i sees key j when j <= i and, if chunk > 0,
 * i / chunk == j / chunk and, if window > 0, i - j < window.  sink [heads] (may be NULL): a term exp(sink[h]) in the
 * denominator of the softmax.  Work is dealt by the tile list, int32 [num_tiles][2] = segment, first row inside it; a tile
 * covers nqh_attention_tile_rows rows.  q [rows, heads, k_row], out [rows, heads * vdim].
 * The positions of every segment must lie inside its block table. */
int64_t nqh_attention_tile_rows(void);
int nqh_attention_prefill(const void* q, const void* k_cache, const void* v_cache, const int32_t* block_tables,
                          const int32_t* segments, const int32_t* tiles, const void* sink, void* out, int64_t rows,
                          int64_t num_tiles, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t k_row,
                          int64_t v_row, int64_t block_size, int64_t max_blocks, int64_t num_blocks, int64_t chunk,
                          int64_t window, float scale, int dtype, void* stream);

/* The same for one new token of each of `batch` sequences: context_lens[b] tokens are cached, the query is the last of
 * them.  block_table int32 [batch, max_blocks].  Workspace: nqh_attention_decode_workspace_bytes, uninitialised. */
size_t nqh_attention_decode_workspace_bytes(int64_t batch, int64_t heads, int64_t kv_heads, int64_t v_row,
                                            int64_t max_context, int64_t chunk, int64_t window, int dtype);
int nqh_attention_decode(const void* q, const void* k_cache, const void* v_cache, const int32_t* block_table,
                         const int32_t* context_lens, const void* sink, void* out, int64_t batch, int64_t heads,
                         int64_t kv_heads, int64_t dim, int64_t vdim, int64_t k_row, int64_t v_row, int64_t block_size,
                         int64_t max_blocks, int64_t num_blocks, int64_t chunk, int64_t window, float scale, int dtype, void* workspace,
                         size_t workspace_bytes, void* stream);

/* Latent attention.  A token's cache row [block][token][row] holds its normalised latent (rank elements) and, at rot_at, the
 * rotated key part (rot_dim) that all heads share; the rest of the row stays zero.
 * nqh_latent_store: proj [rows, heads * (dim + rot_dim) + rank + rot_dim] = the heads' queries [dim | rot_dim], latent,
 * rotated key part.  The latent is RMS-normalised with norm_weight [rank], the rotated parts of queries and key turn pairs
 * (2i, 2i + 1) by cos_sin [max_positions, rot_dim] = cos | sin at positions[row]; latent and key part go to the cache row
 * slots[row] (outside [0, num_slots): not written).  q_out [rows, heads, q_row] receives the rotated part at rot_q and, with
 * copy_plain, the unrotated part at 0; what lies beyond dim (without copy_plain: beyond rank, which nqh_head_linear fills) is
 * zeroed. */
int nqh_latent_store(const void* proj, const void* norm_weight, const float* cos_sin, const int64_t* positions,
                     const int64_t* slots, void* q_out, void* cache, int64_t rows, int64_t heads, int64_t dim,
                     int64_t rot_dim, int64_t rank, int64_t q_row, int64_t rot_q, int copy_plain, int64_t row,
                     int64_t rot_at, int64_t max_positions, int64_t num_slots, float eps, int dtype, void* stream);

/* The contexts of all segments (see nqh_attention_prefill; at most `longest` tokens each) from the cache to consecutive
 * rows without padding: out [., rank + rot_dim], segment s from row first[s] on.  2-byte elements; sizes multiples of 8. */
int nqh_latent_gather(const void* cache, const int32_t* tables, const int32_t* segments, const int32_t* first, void* out,
                      int64_t num_segments, int64_t longest, int64_t rank, int64_t rot_dim, int64_t row, int64_t rot_at,
                      int64_t block_size, int64_t max_blocks, int64_t num_blocks, void* stream);

/* y[r, h, :] = weight[h] x[r, h, :] with weight [heads, out, in]; x_row, x_head, y_row, y_head: elements between rows and
 * between heads. */
int nqh_head_linear(const void* x, const void* weight, void* y, int64_t rows, int64_t heads, int64_t out_features,
                    int64_t in_features, int64_t x_row, int64_t x_head, int64_t y_row, int64_t y_head, int dtype,
                    void* stream);

/* Prompt attention over keys and values expanded per head, bf16: token j of segment s is row first[s] + j of kv [.,
 * kv_stride] = heads x dim unrotated keys, then heads x vdim values, and of rot [., rot_stride], the shared rotated part.
 * q [rows, heads, q_row] with q_row = nqh_latent_attention_prefill_query_row (0: these sizes are not supported); segments and
 * tiles as in nqh_attention_prefill; causal. */
int64_t nqh_latent_attention_prefill_query_row(int64_t dim, int64_t rot_dim, int64_t vdim, int dtype);
int nqh_latent_attention_prefill(const void* q, const void* kv, int64_t kv_stride, const void* rot, int64_t rot_stride,
                                 const int32_t* first, const int32_t* segments, const int32_t* tiles, void* out, int64_t rows,
                                 int64_t num_tiles, int64_t heads, int64_t dim, int64_t rot_dim, int64_t vdim, float scale,
                                 void* stream);

/* Decode attention over the latents themselves: q [batch, heads, row] = queries multiplied into the latent space, with the
 * rotated part at rot_at; out [batch, heads, rank] is still in the latent space.  In bf16 rot_at 64, 128, 256 or 512 with row
 * - rot_at 32 or 64 runs on the matrix cores, anything else (row <= 1024, rank <= 512) on the vector ALU. */
size_t nqh_latent_attention_decode_workspace_bytes(int64_t batch, int64_t heads, int64_t rank, int64_t rot_at, int64_t row,
                                                   int64_t max_context, int dtype);
int nqh_latent_attention_decode(const void* q, const void* cache, const int32_t* block_table, const int32_t* context_lens,
                                void* out, int64_t batch, int64_t heads, int64_t rank, int64_t rot_at, int64_t row,
                                int64_t block_size, int64_t max_blocks, int64_t num_blocks, float scale, int dtype,
                                void* workspace, size_t workspace_bytes, void* stream);

/* Selective scan.  Per channel c and state n: S[n, c] = exp(dt[c] A[c, n]) S[n, c] + dt[c] x[c] B[n], y[c] =
 * (sum_n S[n, c] C[n] + D[c] x[c]) silu(z[c]), A = -exp(a_log [channels, states]).  x is the output of a causal convolution
 * per channel (weight [channels, taps], last column: the current token) with bias and silu.  state fp32 [slots, states,
 * channels], tail fp32 [slots, taps - 1, channels]: the convolution's last inputs, oldest first; neither is ever cleared,
 * before position 0 both count as zero.  bc rows hold B | C.  *_stride: elements between rows.
 * Pieces of a pass as in nqh_gla_prefill (nqh_scan_piece_rows: a good size, the least allowed is what it gives for one row);
 * longest: rows of the longest piece.  At most 256 states and 16 taps. */
int nqh_conv_silu(const void* x, int64_t x_stride, const void* weight, const void* bias, const float* tail,
                  const int32_t* pieces, int64_t num_pieces, int64_t longest, void* out, int64_t channels, int64_t taps,
                  int dtype, void* stream);
int nqh_conv_step(const void* x, int64_t x_stride, const void* weight, const void* bias, float* tail,
                  const int32_t* state_slots, const int64_t* positions, const uint8_t* active, void* out, int64_t batch,
                  int64_t num_slots, int64_t channels, int64_t taps, int dtype, void* stream);
/* dt [rows, channels] = log(1 + exp(weight [channels, rank] low + bias)), fp32. */
int nqh_scan_dt(const void* low, int64_t low_stride, const void* weight, const void* bias, float* dt, int64_t rows,
                int64_t channels, int64_t rank, int dtype, void* stream);
/* The pass's tokens through the recurrence; conv_in: the convolution's inputs, from which the tail is taken.  out [rows,
 * channels].  chained: some sequence has several pieces (the workspace is needed then, uninitialised). */
int64_t nqh_scan_piece_rows(int64_t rows, int64_t channels, int64_t states);
size_t nqh_scan_workspace_bytes(int64_t num_pieces, int64_t channels, int64_t states);
int nqh_scan_prefill(const void* x, const float* dt, const void* bc, int64_t bc_stride, const void* z, int64_t z_stride,
                     const void* a_log, const void* d_skip, const void* conv_in, int64_t conv_stride, float* state, float* tail,
                     const int32_t* pieces, int64_t num_pieces, int chained, void* out, int64_t channels, int64_t states,
                     int64_t taps, int dtype, void* workspace, size_t workspace_bytes, void* stream);
/* One token of each sequence; idle rows and slots as in nqh_gla_decode. */
int nqh_scan_step(const void* x, const float* dt, const void* bc, int64_t bc_stride, const void* z, int64_t z_stride,
                  const void* a_log, const void* d_skip, float* state, const int32_t* state_slots, const int64_t* positions,
                  const uint8_t* active, void* out, int64_t batch, int64_t num_slots, int64_t channels, int64_t states,
                  int dtype, void* stream);

/* decay[r, c] = sigmoid(low[r, :] . up[c, :] + bias[c])^(1 / tau), fp32; low [rows, rank] with row stride low_stride,
 * up [channels, rank]. */
int nqh_gla_decay(const void* low, int64_t low_stride, const void* up, const void* bias, float* decay, int64_t rows,
                  int64_t channels, int64_t rank, float tau, int dtype, void* stream);

/* Gated linear attention over the tokens of a prompt pass.  Per head: S = diag(decay) S + k v^T, o = S^T (q * scale).
 * q, k [rows, heads * dim], v [rows, heads * vdim] with a common row stride; decay [rows, heads * dim] fp32; state fp32
 * [slots, heads, dim, vdim], left as of each sequence's last token; o fp32 [rows, heads * vdim].
 * The pass is a list of pieces, int32 [num_pieces][6] = first row, rows, state slot, whether the sequence starts at zero
 * state, index of the piece in its sequence, pieces of that sequence; the pieces of a sequence are neighbours in order.
 * chained: some sequence has more than one piece (the workspace is needed then, uninitialised).
 * nqh_gla_piece_rows: a good size of pieces for a pass of so many rows. */
int64_t nqh_gla_piece_rows(int64_t rows, int64_t heads, int64_t dim, int64_t vdim);
size_t nqh_gla_prefill_workspace_bytes(int64_t num_pieces, int64_t heads, int64_t dim, int64_t vdim);
int nqh_gla_prefill(const void* q, const void* k, const void* v, int64_t row_stride, const float* decay, float* state,
                    float* o, const int32_t* pieces, int64_t num_pieces, int chained, int64_t heads, int64_t dim,
                    int64_t vdim, float scale, int dtype, void* workspace, size_t workspace_bytes, void* stream);

/* out = RMSNorm(o over each head's vdim) * weight * silu(gate); o fp32 [rows, heads * vdim], gate rows gate_stride
 * apart. */
int nqh_head_norm_gate(const float* o, const void* gate, int64_t gate_stride, const void* weight, void* out, int64_t rows,
                       int64_t heads, int64_t vdim, float eps, int dtype, void* stream);

/* One token of each of `batch` sequences through decay, recurrence, head norm and gate at once.  q, k, v, gate, low:
 * slices of one projection row, row_stride apart; state fp32 [num_slots, heads, dim, vdim], row b uses slot
 * state_slots[b] (zero before position 0); rows with active[b] == 0 or a slot out of range touch no state and give
 * zeros. */
int nqh_gla_decode(const void* q, const void* k, const void* v, const void* gate, const void* low, int64_t row_stride,
                   const void* up, const void* bias, const void* norm_weight, float* state, const int32_t* state_slots,
                   const int64_t* positions, const uint8_t* active, void* out, int64_t batch, int64_t num_slots,
                   int64_t heads, int64_t dim, int64_t vdim, int64_t rank, float tau, float scale, float eps, int dtype,
                   void* stream);

/* scores = sigmoid(router h); per row the `top` experts of largest score (lowest index among equal ones), largest
 * first, and their scores as they are.  h [rows, width], router [experts, width]. */
int nqh_router_topk(const void* h, const void* router, int32_t* expert, float* weight, int64_t rows, int64_t width,
                    int64_t experts, int64_t top, int dtype, void* stream);

/* Groups the pairs (row, choice) -- pair p = row * top + choice -- by expert: order int32 [pairs] lists them expert by
 * expert, and the tile list cuts every expert's run into tiles of at most tile_rows: tiles int32 [3 * max_tiles + 1] =
 * expert[], first place in order[], count[], then the number of tiles.  max_tiles >= nqh_moe_max_tiles. */
int64_t nqh_moe_max_tiles(int64_t pairs, int64_t experts, int64_t tile_rows);
int nqh_moe_plan(const int32_t* expert, int32_t* order, int32_t* tiles, int64_t pairs, int64_t experts, int64_t tile_rows,
                 int64_t max_tiles, void* stream);

/* Experts, both halves over the plan's tiles.  gate_up [experts, 2 * ff, width] (gate rows, then up rows), down
 * [experts, width, ff].
 *   act[place, :] = silu(w (gate h)) * (w (up h)) for the pair order[place], w = weight[pair], h = row pair / top
 *   y[pair, :]    = down act[place]
 * act [pairs, ff] in plan order, y [pairs, width] in pair order.  tile_rows of the plan must be nqh_moe_tile_rows. */
int64_t nqh_moe_tile_rows(int64_t pairs, int64_t experts, int64_t width, int64_t ff, int dtype);
int nqh_moe_gate_up(const void* h, const void* gate_up, const float* weight, const int32_t* order, const int32_t* tiles,
                    void* act, int64_t pairs, int64_t top, int64_t experts, int64_t width, int64_t ff, int64_t tile_rows,
                    int64_t max_tiles, int dtype, void* stream);
int nqh_moe_down(const void* act, const void* down, const int32_t* order, const int32_t* tiles, void* y, int64_t pairs,
                 int64_t experts, int64_t width, int64_t ff, int64_t tile_rows, int64_t max_tiles, int dtype,
                 void* stream);

/* y [rows, out] = act(x [rows, in] weight[out, in]^T (+ bias)) for few rows (<= 64), bf16 operands; y in fp32 if out_f32;
 * act and param as in nqh_activate. */
int nqh_skinny_linear(const void* x, const void* weight, const void* bias, void* y, int64_t rows, int64_t out_features,
                      int64_t in_features, int out_f32, int act, float param, void* stream);

/* Decode-step bookkeeping, as nq_argmax_rows / nq_decode_prepare / nq_decode_advance (nq_engine_ops.h) do it; the
 * logits are fp32. */
int nqh_argmax_rows(const float* logits, int64_t* out, int64_t rows, int64_t vocab, void* stream);
int nqh_decode_prepare(const int64_t* positions, const uint8_t* active, const int32_t* block_table, int64_t* slots,
                       int32_t* context_lens, int64_t rows, int64_t max_blocks, int64_t block_size, void* stream);
int nqh_decode_advance(const int64_t* next_tokens, const uint8_t* active, int64_t* out_log, int64_t* ids,
                       int64_t* positions, int64_t* step, int64_t rows, int64_t out_rows, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* NQ_HYBRID_OPS_H_ */
