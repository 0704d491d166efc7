/*
 * skyrl_layers.h — C ABI of the hybrid decoders' layer libraries (inference_engines/hybrid.py) on MI355X
 * (gfx950): libskyrl_layers.so (embedding, norms, activations, convolutions) and libskyrl_layer_<name>.so for the
 * entry points skyrl_<name>_* of one mechanism, so that serving a model compiles its own kernels only.
 * Conventions (status codes, dtype codes, stream order, no allocation, skyrl_last_error(), one per library) are
 * those of skyrl_hip.h.
 *
 * `dtype` is the element type T of activations and weights: SKYRL_BF16, or SKYRL_F32 for a model run
 * wholly in 32-bit. The residual stream, norms, rotary angles, attention scores and weights, gates
 * and recurrent state are f32 for either.
 */
#ifndef SKYRL_LAYERS_H
#define SKYRL_LAYERS_H

#include "skyrl_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

/* ---- embedding, norms, activations, convolution state, logits ---------------------------------
 *   skyrl_embed     out f32 [n, H] = scale * table T [vocab, H] at tokens i64 [n]. With turns f64 [(H + 1) / 2] the
 *                   position's vector is added: sine (even columns) and cosine (odd) of positions[row] *
 *                   turns[column / 2] revolutions. x T [n, H] (may be NULL): the same rounded.
 *   skyrl_add_norm  hidden f32 [n, H] += delta T [n, H] (may be NULL) and += step T [H] (may be
 *                   NULL: one vector for every row); out T [n, H] = norm(hidden) * (w_base + weight T [H]):
 *                   w_base 0 for a weight stored as it is, 1 for one stored as its distance from 1.
 *                   kind 0: layer norm without bias (mean taken off, variance = mean squared
 *                   deviation), 1: RMS norm; eps inside the root. H <= 8192.
 *   skyrl_norm_add  for sublayers whose output is normed: with rms(v) = v / sqrt(mean(v^2) + eps) over a row of H,
 *                   m = a T [n, H], or, with two outputs, share (rms(a) wa + rms(b) wb) (wa, wb T [H]); hidden f32 +=
 *                   rms(m) * weight; out T = hidden, or rms(hidden) * final_weight if that is given. weight and
 *                   final_weight T hold one number for all columns or H (weight_n, final_n). H <= 8192.
 *   skyrl_gate_norm_add  for sublayers between two norms in `groups` equal parts (norm(v): every part over the root of
 *                   its own mean square + eps): y = the sum of `parts` consecutive rows of H of a, row rows[i] * parts on
 *                   (rows NULL: i * parts), times sigmoid(gate T [n, gate_stride] + gate_bias f32 [H]) if gate is
 *                   given; hidden f32 [n, H] += mult * norm(y) * weight T [H] (fresh: from 0); out T = norm(hidden) *
 *                   next T [H]. H <= 8192.
 *   skyrl_tanh      out T [n, I] = tanh of x T [n, I] (row stride `stride`).
 *   skyrl_gated_norm  out T [n, width] = rms over each of `groups` equal parts of y silu(z), times weight T [width].
 *   skyrl_xielu     out T [n, I] = ap x^2 + x / 2 for x > 0, an (exp(x) - 1 - x) + x / 2 otherwise, ap = softplus(p),
 *                   an = 1/2 + softplus(q) from pq T [2].
 *   skyrl_gate_mul  out T [n, I] (row stride out_stride) from gate | up of gate_up T [n, 2I] (row stride
 *                   gu_stride): act 0: silu(gate) * up, 1: gelu(gate) * up in gelu's tanh form, 2: with
 *                   g = min(gate, limit) and u = up clamped to +-limit, g * sigmoid(alpha g) * (u + 1).
 *                   f32 throughout, rounded once. alpha and limit are of act 2.
 *   skyrl_conv_save stores the last `taps` rows of every sequence's columns [0, channels) of x T [T, stride]
 *                   in ring T [rows, taps, channels], the row of position p at p % taps. Sequences: tokens
 *                   [cu[s], cu[s+1]) of row rows[s] (< 0: skipped), positions consecutive from positions[cu[s]].
 *   skyrl_softcap   out f32 = cap * tanh(x / cap) over count elements of x T (cap <= 0: a copy). */
#define SKYRL_NORM_LAYER 0
#define SKYRL_NORM_RMS 1
#define SKYRL_ACT_SILU 0
#define SKYRL_ACT_GELU_TANH 1
#define SKYRL_ACT_CLAMPED 2
int skyrl_embed(const int64_t* tokens, const void* table, int64_t n, int32_t H, float scale, const int64_t* positions,
                const double* turns, float* out, void* x, int32_t dtype, void* stream);
int skyrl_norm_add(const void* a, const void* wa, const void* b, const void* wb, float share, float* hidden,
                   const void* weight, int32_t weight_n, const void* final_weight, int32_t final_n, int32_t n,
                   int32_t H, float eps, void* out, int32_t dtype, void* stream);
int skyrl_xielu(const void* x, int64_t stride, int64_t n, int32_t I, const void* pq, void* out, int64_t out_stride,
                int32_t dtype, void* stream);
int skyrl_add_norm(const void* delta, float* hidden, const void* step, const void* weight, float w_base, int32_t n,
                   int32_t H, float eps, int32_t kind, void* out, int32_t dtype, void* stream);
int skyrl_gated_norm(const void* y, int64_t y_stride, const void* z, int64_t z_stride, const void* weight, int64_t n,
                     int32_t width, int32_t groups, float eps, void* out, int64_t out_stride, int32_t dtype,
                     void* stream);
int skyrl_gate_mul(const void* gate_up, int64_t gu_stride, int64_t n, int32_t I, int32_t act, float alpha, float limit,
                   void* out, int64_t out_stride, int32_t dtype, void* stream);
int skyrl_gate_norm_add(const void* a, const int64_t* rows, int32_t parts, const void* gate, int64_t gate_stride,
                        const float* gate_bias, const void* weight, int32_t groups, float eps, float mult, float* hidden,
                        int32_t fresh, const void* next, int32_t n, int32_t H, void* out, int32_t dtype, void* stream);
int skyrl_tanh(const void* x, int64_t stride, int64_t n, int32_t I, void* out, int32_t dtype, void* stream);
int skyrl_conv_save(const void* x, int64_t stride, int32_t channels, int32_t taps, const int32_t* cu,
                    const int32_t* rows, const int64_t* positions, int32_t nseq, void* ring, int32_t dtype,
                    void* stream);
int skyrl_softcap(const void* x, float* out, int64_t count, float cap, int32_t dtype, void* stream);

/* ---- latent attention over a paged latent cache ----------------------------------------------
 * A layer run's cache is T [num_blocks, 16, row]: per token the normed latent (rank), the rotated key
 * part all heads share (rot_dim), zero padding up to row = a multiple of 32. slot = block * 16 +
 * offset. Token t of a step belongs to row bt_row[t] of block_tables i32 [*, bt_stride] and attends
 * to the cached positions [max(0, positions[t] - window + 1), positions[t]] (window <= 0: all).
 * Rotations pair neighbouring dimensions, or with `halves` i and i + rot_dim / 2; cos_sin f32 [max_pos, rot_dim] =
 * cos | sin halves, one entry per pair, amplitude included. sinks f32 [heads] (may be NULL): exp(sink) joins a
 * head's denominator. gate T [T, gate_stride] (may be NULL): a head's output times sigmoid(gate[t][head]).
 *   skyrl_latent_write   rows of proj T [T, proj_stride], in place, each part optional: heads > 0: q (heads x (dim +
 *                        rot_dim)) at the row's start, its rotated parts turned; q_rank > 0: a query latent there,
 *                        RMS-normed (weight T [q_rank]); rank > 0: at latent_at the key latent (rank) | key part
 *                        (rot_dim), RMS-normed (weight T [rank]) and turned into the cache at slots[t] (< 0: no write).
 *   skyrl_latent_attend  one query row per token in the latent space: qa T [heads, T, rank] is the
 *                        unrotated query times the key up-projection, q_rot points at the rotated part
 *                        of head 0 of token 0 (token stride q_stride, head stride q_head); out
 *                        T [heads, T, rank] = softmax(scale * (qa.c + q_rot.k_rot)) c. nparts
 *                        workgroups share a token's keys (MFMA form, bf16); part_min >= 16 keys, a
 *                        multiple of 16, per workgroup; nparts > 1 needs skyrl_latent_attend_workspace_bytes. f32, and
 *                        shapes outside the MFMA form (skyrl_latent_attend_mfma == 0), take a plain
 *                        kernel and ignore nparts.
 *   skyrl_latent_gather  prompt form, step 1: copies for each of nseg segments the cached rows of
 *                        positions [seg_first, seg_first + seg_count) (seg i32 [nseg, 4]: block-table
 *                        row, first position, count, first packed row) to latent T [rows, rank] and
 *                        k_rot T [rows, rot_dim].
 *   skyrl_latent_prefill prompt form, step 2 (bf16): per head keys k_nope [rows, k_stride] (head h at
 *                        h * dim) | k_rot, values transposed v_t [heads * vdim, vt_stride] over packed
 *                        rows; one workgroup per (tile, head), tiles i32 [ntiles, 8]: first token,
 *                        token count (<= 128), position of the first token, first packed row of its
 *                        segment, position of that row, 0, 0, 0. A segment's packed rows are a multiple
 *                        of 64 (skyrl_latent_gather zeroes the padding rows). out T [T, out_stride], head h at
 *                        h * vdim. dim + rot_dim <= 256, vdim <= 256, vt_stride % 64 == 0. */
int skyrl_latent_write(void* proj, int64_t proj_stride, int32_t T, int32_t heads, int32_t dim, int32_t rot_dim,
                       int32_t halves, int32_t q_rank, const void* q_norm, int32_t rank, int32_t latent_at,
                       const void* norm_weight, float eps, const int64_t* positions, const int64_t* slots,
                       const float* cos_sin, void* cache, int32_t row, int32_t dtype, void* stream);
int skyrl_latent_attend_mfma(int32_t rank, int32_t rot_dim, int32_t row, int32_t dtype);
size_t skyrl_latent_attend_workspace_bytes(int32_t T, int32_t heads, int32_t rank, int32_t nparts);
int skyrl_latent_attend(const void* qa, const void* q_rot, int64_t q_stride, int64_t q_head, const void* cache,
                        int32_t row, const int32_t* block_tables, int64_t bt_stride, const int32_t* bt_row,
                        const int64_t* positions, int32_t T, int32_t heads, int32_t rank, int32_t rot_dim,
                        float scale, int32_t window, int32_t part_min, int32_t nparts, const float* sinks,
                        const void* gate, int64_t gate_stride, void* out, void* workspace, int32_t dtype, void* stream);
int skyrl_latent_gather(const void* cache, int32_t row, const int32_t* block_tables, int64_t bt_stride,
                        const int32_t* seg, int32_t nseg, int32_t max_count, int32_t rank, int32_t rot_dim,
                        void* latent, void* k_rot, int32_t dtype, void* stream);
int skyrl_latent_prefill(const void* q, int64_t q_stride, const void* k_nope, int64_t k_stride, const void* k_rot,
                         const void* v_t, int64_t vt_stride, const int32_t* tiles, int32_t ntiles, int32_t heads,
                         int32_t dim, int32_t rot_dim, int32_t vdim, float scale, int32_t window, const float* sinks,
                         const void* gate, int64_t gate_stride, void* out, int64_t out_stride, void* stream);

/* ---- gated delta rule ------------------------------------------------------------------------
 * proj T [T, proj_stride]: q (kv_heads x dim) | k (kv_heads x dim) | v (heads x vdim) | output gate
 * (heads x vdim) | beta (heads) | decay (heads). q, k and v pass a causal convolution over time
 * (conv_w T [2 kv_heads dim + heads vdim, taps], last tap on the current token) and silu; q and k
 * become unit vectors, q times dim^-1/2. Per head: S <- g S; u = sigmoid(beta) (v - S^T k); S <- S +
 * k u^T; o = S^T q with g = exp(-exp(A_log) softplus(decay + dt_bias)); out = rms_norm(o) * norm_w *
 * silu(output gate).
 * State per row: S f32 [rows, heads, dim, vpad], vpad = vdim up to a multiple of 4, and the last
 * `taps` inputs of the convolutions, T [rows, taps, channels], the input of position p at p % taps. A
 * sequence that starts at position 0 starts from zero, whatever the row holds.
 * Sequences: tokens [cu[s], cu[s+1]) of row rows[s] (< 0: skipped, nothing written), their positions
 * consecutive from positions[cu[s]].
 *   skyrl_delta_scan       token by token, the state in registers: decode steps and short portions.
 *                          save_conv 1 also stores the convolution inputs and needs every sequence to
 *                          have one token; otherwise skyrl_conv_save of the channels follows.
 *   Prompt form, for portions of many tokens, in chunks of 64: chunk i32 [nchunks, 4] (first token,
 *   tokens <= 64, sequence, 0), chunks of one sequence consecutive and in order, cut from its first
 *   token on; d16, v16 = dim, vdim up to a multiple of 16. dim <= 256.
 *   skyrl_delta_conv       1: qk f32 [T, 2, kv_heads, d16] (unit vectors, q scaled), kt f32
 *                          [nchunks, kv_heads, d16, 64] (k transposed), v f32 [T, heads, vdim], lg f32 [T, heads] (log decay), beta f32 [T, heads], at the
 *                          chunks' tokens.
 *   skyrl_delta_chunk      2: each chunk's own triangular system: W f32 [nchunks, heads, 64, d16],
 *                          U f32 [nchunks, heads, v16, 64] (transposed), P f32 [nchunks, heads, 64, 64] (its
 *                          blocks below and on the diagonal), G f32
 *                          [nchunks, heads, 64] (summed log decays).
 *   skyrl_delta_chain      3: sequential over the chunks seq_chunks[i] .. seq_chunks[i + 1] - 1 of sequence
 *                          seq0 + i: reads and writes S, o f32 [T, heads, vdim]. skyrl_conv_save stores
 *                          the convolution inputs.
 *   skyrl_delta_out        4: out T of tokens [first, T) from o. */
typedef struct skyrl_delta_shape {
    int32_t heads, kv_heads, dim, vdim, taps;
    float eps; /* of the output norm */
} skyrl_delta_shape;
int skyrl_delta_scan(const skyrl_delta_shape* shape, const void* proj, int64_t proj_stride, const void* conv_w,
                     const float* a_log, const float* dt_bias, const void* norm_w, const int32_t* cu,
                     const int32_t* rows, const int64_t* positions, int32_t nseq, float* state, void* conv_state,
                     int32_t save_conv, void* out, int64_t out_stride, int32_t dtype, void* stream);
int skyrl_delta_conv(const skyrl_delta_shape* shape, const void* proj, int64_t proj_stride, const void* conv_w,
                     const float* a_log, const float* dt_bias, const int32_t* chunk, int32_t nchunks,
                     const int32_t* cu, const int32_t* rows, const int64_t* positions, const void* conv_state,
                     float* qk, float* kt, float* v, float* lg, float* beta, int32_t dtype, void* stream);
int skyrl_delta_chunk(const skyrl_delta_shape* shape, const int32_t* chunk, int32_t nchunks, const float* qk,
                      const float* v, const float* lg, const float* beta, float* W, float* U, float* P, float* G,
                      void* stream);
int skyrl_delta_chain(const skyrl_delta_shape* shape, const int32_t* chunk, const int32_t* seq_chunks, int32_t seq0,
                      int32_t nseq, const int32_t* cu, const int32_t* rows, const int64_t* positions, const float* qk,
                      const float* kt, const float* W, const float* U, const float* P, const float* G, float* state, float* o,
                      void* stream);
int skyrl_delta_out(const skyrl_delta_shape* shape, const float* o, const void* proj, int64_t proj_stride,
                    const void* norm_w, int32_t first, int32_t T, void* out, int64_t out_stride, int32_t dtype,
                    void* stream);

/* ---- differential attention over a paged key / value cache -------------------------------------
 * A query head has two maps, each an attention of its own over the same values: a_m = softmax(scale
 * q_m . k_m) v, o = a_1 - lambda a_2, out = o / rms(o) (1 - diff) sigmoid(gate), the root mean square (eps
 * inside) over the head's vdim values. Query head h reads key / value head h / (heads / kv_heads).
 * proj T [T, proj_stride]: q (heads x 2 x dim) | k (kv_heads x 2 x dim) | v (kv_heads x vdim), with k and v
 * only if `kv` (else the keys and values are another layer's, in its cache). Each channel passes a causal
 * convolution over time (conv_t f32 [taps, channels], last tap on the current token; state as under
 * skyrl_conv_save), then the first rot_dims of every map of q and k are rotated (interleaved pairs;
 * cos_sin f32 [max_pos, rot_dims] = cos | sin halves, amplitude included).
 * Padded sizes: dp = dim up to a multiple of 16, vp = vdim likewise. Queries T [T, heads, 2 dp], map m
 * from m dp on, zeros between. Cache: keys T [num_blocks, kv_heads, 16, 2 dp], values transposed T
 * [num_blocks, kv_heads, vp, 16]; padding must hold zeros. slot = block * 16 + offset. Token t of a
 * step belongs to row bt_row[t] of block_tables, which is also its sequence (cu, rows), and attends to
 * positions [0, positions[t]].
 *   skyrl_diff_write      tokens [first, first + count): convolution, rotation, queries out, keys and values
 *                         into the cache at slots[t] (< 0: no write). save_conv 1 also stores the
 *                         convolution inputs and needs every sequence to have one token; otherwise
 *                         skyrl_conv_save follows. Padding is not written.
 *   skyrl_diff_write_runs the same (bf16, dim and vdim multiples of 8, taps <= 8) by runs i32 [nruns, 2]: first
 *                         token, count <= 8 of one sequence, whose slots lie in one half of a block.
 *   skyrl_diff_attend     one query row per token; gate T points at head 0 of token 0 (row stride
 *                         gate_stride); lambda f32 [1]; out T (row stride out_stride), head h at h * vdim.
 *                         nparts waves share a token's keys (MFMA form, bf16), each at least part_min >= 16
 *                         keys, a multiple of 16; nparts > 1 needs skyrl_diff_attend_workspace_bytes. f32, and
 *                         shapes outside the MFMA form (skyrl_diff_mfma == 0), take a plain kernel and
 *                         ignore nparts.
 *   skyrl_diff_prefill    prompt form (bf16, skyrl_diff_mfma != 0): one workgroup per (tile, head); tiles i32
 *                         [ntiles, 4]: first token, token count (<= 128), position of the first token, row
 *                         of block_tables. */
typedef struct skyrl_diff_shape {
    int32_t heads, kv_heads, dim, vdim, rot_dims, taps, kv;
    float scale, diff, eps;
} skyrl_diff_shape;
int skyrl_diff_write(const skyrl_diff_shape* shape, const void* proj, int64_t proj_stride, const float* conv_t,
                     const int32_t* cu, const int32_t* rows, const int32_t* bt_row, const int64_t* positions,
                     const int64_t* slots, const float* cos_sin, void* ring, int32_t save_conv, int32_t first,
                     int32_t count, void* q, void* k_cache, void* v_cache, int32_t dtype, void* stream);
int skyrl_diff_write_runs(const skyrl_diff_shape* shape, const void* proj, int64_t proj_stride, const float* conv_t,
                          const int32_t* cu, const int32_t* rows, const int32_t* bt_row, const int64_t* positions,
                          const int64_t* slots, const float* cos_sin, const void* ring, const int32_t* runs,
                          int32_t nruns, void* q, void* k_cache, void* v_cache, void* stream);
int skyrl_diff_mfma(const skyrl_diff_shape* shape, int32_t dtype);
size_t skyrl_diff_attend_workspace_bytes(const skyrl_diff_shape* shape, int32_t T, int32_t nparts);
int skyrl_diff_attend(const skyrl_diff_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                      const void* k_cache, const void* v_cache, const int32_t* block_tables, int64_t bt_stride,
                      const int32_t* bt_row, const int64_t* positions, int32_t T, const float* lambda,
                      int32_t part_min, int32_t nparts, void* out, int64_t out_stride, void* workspace, int32_t dtype,
                      void* stream);
int skyrl_diff_prefill(const skyrl_diff_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                       const void* k_cache, const void* v_cache, const int32_t* block_tables, int64_t bt_stride,
                       const int32_t* tiles, int32_t ntiles, const float* lambda, void* out, int64_t out_stride,
                       void* stream);

/* ---- short convolutions of a prompt's tokens ---------------------------------------------------
 * Causal convolution of columns [0, channels) of x T [T, stride] (conv_t f32 [taps, channels], last tap on the
 * current token; inputs before the step from the ring as under skyrl_conv_save, zero before position 0), plus
 * bias f32 [channels] (may be NULL), then the activation, at the tokens of chunks i32 [nchunks, 4] (first token,
 * tokens <= 64, sequence, 0). Consecutive sections of the channels, each units x size, go to rows T [T, units,
 * padded] and / or transposed to cols T [nchunks, units, padded, 64], zero past a chunk's end (either may be NULL;
 * padding is not written). */
#define SKYRL_CONV_NONE 0
#define SKYRL_CONV_SILU 1
typedef struct skyrl_conv_section {
    int32_t units, size, padded;
    void *rows, *cols;
} skyrl_conv_section;
int skyrl_conv_chunk(const void* x, int64_t stride, int32_t channels, int32_t taps, const float* conv_t,
                     const float* bias, int32_t act, const int32_t* chunk, int32_t nchunks, const int32_t* cu,
                     const int32_t* rows, const int64_t* positions, const void* ring,
                     const skyrl_conv_section* sections, int32_t nsections, int32_t dtype, void* stream);

/* ---- gated linear recurrence (RG-LRU) ----------------------------------------------------------
 * proj T [T, proj_stride]: output gate y (width) | recurrence input (width). u = the input's short convolution
 * plus bias. With u cut into `blocks` equal parts, r and i = sigmoid(W u + b) per part; log a = rate r; S <- a S +
 * sqrt(1 - a^2) i u per channel; out = S gelu(y) (tanh form). gate_w T [blocks, 2 (r, i), np, kp] zero-padded (np, kp:
 * a part's size up to a multiple of 16, of 32), gate_b f32 [2, width], rate f32 [width].
 * State per row: S f32 [rows, width] and the convolution's ring T [rows, taps, width]. A sequence that starts at
 * position 0 starts from zero, whatever the row holds.
 *   skyrl_rglru_step    decode: token s is the one token of sequence s, row rows[s] (< 0: skipped).
 *   skyrl_rglru_prompt  u T [T, width] from skyrl_conv_chunk; chunks as there, their fourth number the run they belong
 *                       to; runs i32 [nruns, 4]: first chunk, chunks, sequence, unused; seq_runs[i] .. seq_runs[i + 1]
 *                       - 1 those of sequence seq0 + i. Scratch: hbuf, abuf f32 [T, width], s_in f32 [nruns, width].
 *                       skyrl_conv_save stores the ring. */
int skyrl_rglru_step(const void* proj, int64_t proj_stride, int32_t width, int32_t blocks, int32_t taps,
                     const float* conv_t, const float* conv_b, const void* gate_w, const float* gate_b,
                     const float* rate, const int32_t* rows, const int64_t* positions, int32_t n, float* state,
                     void* ring, void* out, int64_t out_stride, int32_t dtype, void* stream);
int skyrl_rglru_prompt(const void* proj, int64_t proj_stride, int32_t width, int32_t blocks, const void* u,
                       const void* gate_w, const float* gate_b, const float* rate, const int32_t* chunk,
                       int32_t nchunks, const int32_t* runs, int32_t nruns, const int32_t* seq_runs, int32_t seq0,
                       int32_t nseq, const int32_t* cu, const int32_t* rows, const int64_t* positions, float* state, float* hbuf, float* abuf,
                       float* s_in, void* out, int64_t out_stride, int32_t dtype, void* stream);

/* ---- grouped attention with normed queries and keys, a window and an output gate ---------------
 * proj T [T, proj_stride]: q (heads x dim) | k (kv_heads x dim) | v (kv_heads x vdim). q and k are RMS-normed per
 * head (weights T [dim]); out = softmax(scale q . k) v over the positions [max(0, pos - window + 1), pos] (window
 * <= 0: all) times sigmoid(gate), gate T of the output's layout. Query head h reads key / value head h / (heads /
 * kv_heads). dp = dim up to a multiple of 32, vp = vdim to one of 16: queries T [T, heads, dp], keys T [num_blocks,
 * kv_heads, 16, dp], values transposed T [num_blocks, kv_heads, vp, 16]; padding must hold zeros and is not
 * written. slot = block * 16 + offset; token t belongs to row bt_row[t] of block_tables.
 *   skyrl_attn_write    tokens [first, first + count), or, with runs i32 [count, 2] (first token, tokens <= 8 of one
 *                       sequence whose slots lie in one half of a block; bf16, dim and vdim multiples of 8), those.
 *                       Keys and values go to slots[t] (< 0: no write).
 *   skyrl_attn_attend   one query row per token. nparts waves share a token's keys (MFMA form, bf16), each at least
 *                       part_min >= 16 keys, a multiple of 16; nparts > 1 needs skyrl_attn_attend_workspace_bytes. f32,
 *                       and shapes outside the MFMA form (skyrl_attn_mfma == 0), take a plain kernel and ignore nparts.
 *   skyrl_attn_prefill  prompt form (bf16, skyrl_attn_mfma != 0): one workgroup per (tile, head); tiles i32 [ntiles, 4]:
 *                       first token, token count (<= 128), position of the first token, row of block_tables. */
typedef struct skyrl_attn_shape {
    int32_t heads, kv_heads, dim, vdim, window;
    float scale, eps;
} skyrl_attn_shape;
int skyrl_attn_write(const skyrl_attn_shape* shape, const void* proj, int64_t proj_stride, const void* q_norm,
                     const void* k_norm, const int64_t* slots, const int32_t* runs, int32_t first, int32_t count,
                     void* q, void* k_cache, void* v_cache, int32_t dtype, void* stream);
int skyrl_attn_mfma(const skyrl_attn_shape* shape, int32_t dtype);
size_t skyrl_attn_attend_workspace_bytes(const skyrl_attn_shape* shape, int32_t T, int32_t nparts);
int skyrl_attn_attend(const skyrl_attn_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                      const void* k_cache, const void* v_cache, const int32_t* block_tables, int64_t bt_stride,
                      const int32_t* bt_row, const int64_t* positions, int32_t T, int32_t part_min, int32_t nparts,
                      void* out, int64_t out_stride, void* workspace, int32_t dtype, void* stream);
int skyrl_attn_prefill(const skyrl_attn_shape* shape, const void* q, const void* gate, int64_t gate_stride,
                       const void* k_cache, const void* v_cache, const int32_t* block_tables, int64_t bt_stride,
                       const int32_t* tiles, int32_t ntiles, void* out, int64_t out_stride, void* stream);

/* ---- state space mixer (Mamba-2) ----------------------------------------------------------------
 * proj T [T, proj_stride]: z (heads x vdim) | x (heads x vdim) | B (groups x state) | C (groups x state) | dt
 * (heads). x, B and C pass a short convolution with bias and silu. Head h with group h / (heads / groups): dt =
 * softplus(dt + dt_bias); S <- exp(-exp(A_log) dt) S + dt B x^T; y = S^T C + skip x.
 * State per row: S f32 [rows, heads, state, ppad], ppad = vdim up to a multiple of 4, and the convolution's ring T
 * [rows, taps, heads vdim + 2 groups state]. A sequence that starts at position 0 starts from zero.
 *   skyrl_ssd_scan    token by token over each sequence's tokens [cu[s], cu[s+1]) (row rows[s] < 0: skipped); y T.
 *                     save_conv 1 also stores the convolution inputs and needs every sequence to have one token;
 *                     otherwise skyrl_conv_save follows.
 *   skyrl_ssd_prompt  bf16, state <= 256, from skyrl_conv_chunk's outputs: xt [nchunks, heads, vp, 64], bt [nchunks,
 *                     groups, np, 64], brow and crow [T, groups, np] (vp, np: vdim, state up to a multiple of 16, of
 *                     32; padding zero). super i32 [nsuper, 4]: first chunk, chunks, sequence, 1 if the sequence has
 *                     several such runs + 2 if its last; pick i32 [npick]: the runs that are followed by another of
 *                     their sequence; chain i32 [nchain, 2]: first run and number of runs of the sequences with
 *                     several. Scratch: scores f32 [nchunks, groups, 10, 256], runs f32 [nsuper, heads, np, vp], gtot f32 [nsuper, heads]. */
typedef struct skyrl_ssd_shape {
    int32_t heads, vdim, state, groups, taps;
} skyrl_ssd_shape;
int skyrl_ssd_scan(const skyrl_ssd_shape* shape, const void* proj, int64_t proj_stride, const float* conv_t,
                   const float* conv_b, const float* a_log, const float* dt_bias, const float* skip, const int32_t* cu,
                   const int32_t* rows, const int64_t* positions, int32_t nseq, float* state, void* ring,
                   int32_t save_conv, void* y, int64_t y_stride, int32_t dtype, void* stream);
int skyrl_ssd_prompt(const skyrl_ssd_shape* shape, const void* xt, const void* bt, const void* brow, const void* crow,
                     const void* dt_raw, int64_t dt_stride, const float* a_log, const float* dt_bias,
                     const float* skip, const int32_t* chunk, int32_t nchunks, const int32_t* super,
                     int32_t nsuper, const int32_t* pick, int32_t npick, const int32_t* chain, int32_t nchain,
                     const int32_t* cu, const int32_t* rows, const int64_t* positions, float* state, float* scores,
                     float* runs, float* gtot, void* y, int64_t y_stride, void* stream);

/* ---- generalized delta rule ------------------------------------------------------------------------
 * proj T [T, proj_stride]: r | k | v | output gate | removal rate, each heads x dim; wl T [T, wl_stride] the decay
 * logits (heads x dim); w0, a_bias f32 [heads dim]; norm_w T [heads dim]. Per head, with u = k / sqrt(sum k^2 + 1e-6),
 * w = exp(-e^(-1/2) sigmoid(wl + w0)) and a = sigmoid(removal rate + a_bias), S the state before the token:
 *   S' = diag(w) S - (a u) (u^T S) + k v^T;  o = S'^T r;  out = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(output gate).
 * State per row: f32 [rows, heads, dim, vpad], vpad = dim up to a multiple of 4. Sequences, rows and chunks as for the
 * gated delta rule. dim <= 256.
 *   skyrl_gdelta_scan   token by token, the state in registers: decode steps and short portions.
 *   Prompt form, chunks of 64, d16 = dim up to a multiple of 16, all f32:
 *   skyrl_gdelta_chunk  1: what a chunk does to the state, S <- M S + N, and its outputs O + R S: M [nchunks, heads, d16,
 *                       d16], N [.., d16 values, d16 keys], R and O [.., 64, d16].
 *   skyrl_gdelta_chain  2: sequences seq0.. of nseq: the states along each sequence's chunks [seq_chunks[i], seq_chunks[i
 *                       + 1]), updated in `state`, every chunk's first one in first [nchunks, heads, d16 values, d16 keys].
 *   skyrl_gdelta_out    3: outputs, head norm, weight and gate (gate T [T, gate_stride]: proj's output gate columns). */
typedef struct {
    int32_t heads, dim;
    float eps;
} skyrl_gdelta_shape;
int skyrl_gdelta_scan(const skyrl_gdelta_shape* shape, const void* proj, int64_t proj_stride, const void* wl,
                      int64_t wl_stride, const float* w0, const float* a_bias, const void* norm_w, const int32_t* cu,
                      const int32_t* rows, const int64_t* positions, int32_t nseq, float* state, void* out,
                      int64_t out_stride, int32_t dtype, void* stream);
int skyrl_gdelta_chunk(const skyrl_gdelta_shape* shape, const void* proj, int64_t proj_stride, const void* wl,
                       int64_t wl_stride, const float* w0, const float* a_bias, const int32_t* chunk, int32_t nchunks,
                       float* M, float* N, float* R, float* O, int32_t dtype, void* stream);
int skyrl_gdelta_chain(const skyrl_gdelta_shape* shape, const int32_t* chunk, const int32_t* seq_chunks, int32_t seq0,
                       int32_t nseq, const int32_t* cu, const int32_t* rows, const int64_t* positions, const float* M,
                       const float* N, float* state, float* first, void* stream);
int skyrl_gdelta_out(const skyrl_gdelta_shape* shape, const int32_t* chunk, int32_t nchunks, const float* R,
                     const float* O, const float* first, const void* gate, int64_t gate_stride, const void* norm_w,
                     void* out, int64_t out_stride, int32_t dtype, void* stream);

/* ---- routed experts ------------------------------------------------------------------------------------
 * x T [n, width]. Of `experts` gated feed-forwards (gate_up T [experts, 2, ff, width], down T [experts, width, ff])
 * each token runs `top`: scores s = sigmoid(router x) (router T [experts, width], f32 sums), choice scores s +
 * correction f32 [experts]; of `groups` equal groups of neighbours the `keep` with the largest sum of their two largest
 * choice scores may be chosen from; the `top` largest of those are, ties to the lower index. Pair p = token * top + i.
 *   skyrl_moe_route    idx i32 [n, top], weight f32 [n, top] (the scores s of the chosen).
 *   skyrl_moe_tiles    the most tiles of tm rows that npairs pairs can fill.
 *   skyrl_moe_sort     pairs by expert: order i32 [ntiles, tm] (pair, or -1), tile_expert i32 [ntiles + 1] (-1: unused; the
 *                      last: tiles in use). counts: scratch of skyrl_moe_counts(experts, npairs) i32 (0: NULL).
 *   skyrl_moe_gate_up  act T [ntiles tm, ff], by sorted place = silu(gate x) * up x. tm a multiple of 16; 16, 64, 128 and
 *                      256 have a matrix form (bf16, width and ff multiples of 8).
 *   skyrl_moe_down     out T [n top, width], by pair = weight * down act. */
typedef struct {
    int32_t width, ff, experts, top, groups, keep;
} skyrl_moe_shape;
int skyrl_moe_route(const skyrl_moe_shape* shape, const void* x, int32_t n, const void* router, const float* correction,
                    int32_t* idx, float* weight, int32_t dtype, void* stream);
int32_t skyrl_moe_tiles(int32_t experts, int32_t npairs, int32_t tm);
int32_t skyrl_moe_counts(int32_t experts, int32_t npairs);
int skyrl_moe_sort(const int32_t* idx, int32_t npairs, int32_t experts, int32_t tm, int32_t ntiles, int32_t* counts,
                   int32_t* order, int32_t* tile_expert, void* stream);
int skyrl_moe_gate_up(const skyrl_moe_shape* shape, const void* x, const void* w, const int32_t* order,
                      const int32_t* tile_expert, int32_t tm, int32_t ntiles, void* act, int32_t dtype, void* stream);
int skyrl_moe_down(const skyrl_moe_shape* shape, const void* act, const void* w, const int32_t* order,
                   const int32_t* tile_expert, int32_t tm, int32_t ntiles, const float* weight, void* out, int32_t dtype,
                   void* stream);

#ifdef __cplusplus
}
#endif
#endif /* SKYRL_LAYERS_H */
