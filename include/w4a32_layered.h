/*
 * C ABI of the layered decoder: a decoder-only model whose layers are described one by one (kind of token mixer,
 * its sizes, feed-forward or none), with unquantised weights in bf16 or f32. It serves designs the Qwen2 runner of
 * w4a32_decoder.h has no operators for: pooled-window attention, the gated delta rule, retention, layer norm with
 * an input convolution, PolyNorm feed-forward; rotary attention with sinks, latent attention, mixtures of experts and
 * layers that run several times in a row.
 *
 * Same conventions as w4a32_hip.h: d_* pointers are device memory, calls only enqueue on `stream`, nothing
 * allocates, synchronises or exits; the return value is a W4A32_* code. The position lives in device memory, so
 * a decode step is one fixed launch sequence that may be captured into a HIP graph and replayed per token.
 *
 * Notation of the mechanisms (t: token, p: its position in the sequence, everything causal):
 *   input convolution    y_t = h_t + sum_j w_j * h_(t - taps + 1 + j), per channel, h = layer norm (weight, no bias)
 *   pooled window        a query attends to the last `window` tokens (itself included) and, in the same softmax, to
 *                        the mean key / value of every complete block of `pool` tokens the window has left behind
 *   gated delta rule     S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
 *   retention            S <- decay S + k v^T;  o = S^T q
 *   PolyNorm             a N(z) + b N(z^2) + c N(z^3) + e, N = division by the root mean square of the token's vector
 *   rotary attention     causal softmax attention on rotated q and k, over the last `window` tokens or all of them; a
 *                        sink adds exp(sink) to a head's softmax denominator; the values may be the unrotated keys
 *   latent attention     a token leaves a normed latent c [kv_rank] and one rotated key part [rot_part] for all heads;
 *                        head h scores (q_h . U_h c + qr_h . kr) * scale and reads the values V_h c. Prefill expands keys
 *                        and values from the cached latents, decoding folds U_h into the query and V_h into the output
 *   mixture of experts   the `top` experts with the largest router logits, weighted by the softmax over those logits;
 *                        expert: down(g sigmoid(1.702 g) (u + 1)), g = min(gate(h), limit), u = clamp(up(h), +-limit)
 *   loop                 layers [loop_start, loop_stop) run loop_times times in a row on the same weights, each pass with
 *                        caches of its own and with x <- W_in [x; x_0] in front, x_0 the embedding row
 *
 * "T" below is the model's element type: bf16 (W4A32_LAYERED_BF16) or f32 (W4A32_LAYERED_F32). In both, the
 * residual stream, norms, scores, softmax, recurrent state and everything that enters a recurrence are f32; with
 * bf16 the matrices, the rows that enter a matrix product and the key / value caches are bf16 (f32 accumulation).
 *
 * Padded sizes: pad(n) = n rounded up to a multiple of 64. Matrices are [pad(out)][pad(in)], vectors over channels
 * [pad(n)], all padding zero; only the embedding and the head keep their true number of rows (vocab).
 */
#ifndef W4A32_LAYERED_H
#define W4A32_LAYERED_H

#include "w4a32_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

#define W4A32_LAYERED_BF16 1
#define W4A32_LAYERED_F32 2

#define W4A32_MIX_ATTENTION 1
#define W4A32_MIX_DELTA 2
#define W4A32_MIX_RETENTION 3
#define W4A32_MIX_ROTARY 4
#define W4A32_MIX_LATENT 5

#define W4A32_NORM_LAYER 0 /* layer norm, always with the input convolution */
#define W4A32_NORM_RMS 1   /* x / sqrt(mean(x^2) + eps) * w, input convolution optional */

#define W4A32_LAYERED_MAX_TAPS 8 /* longest short convolution and input convolution */
#define W4A32_LAYERED_MAX_DIM 256 /* largest dim and vdim of a head */
#define W4A32_LAYERED_MAX_LATENT 512 /* largest kv_rank */
#define W4A32_LAYERED_MAX_ROT_PART 128
#define W4A32_LAYERED_MAX_EXPERTS 512
#define W4A32_LAYERED_MAX_TOP 16
#define W4A32_LAYERED_PAD 64

typedef struct {
  int mixer;                /* W4A32_MIX_* */
  int heads, kv_heads;      /* kv_heads: key / value heads (attention), query / key heads (delta); = heads (retention) */
  int dim, vdim;            /* size of a query / key head and of a value head */
  int conv_taps;            /* attention, delta: taps of the short convolution on q, k, v; 0: none (attention only) */
  float scale;              /* attention, rotary, latent: factor of the scores */
  int window, pool;         /* attention; window also rotary, latent (0: every token) */
  int kv_from;              /* attention: -1, or the earlier attention layer whose keys and values this one reads */
  int rot_dims;             /* retention, rotary, latent: rotated dimensions of a head (even; 0: none) */
  double rot_base;
  int ff;                   /* feed-forward width (of one expert), 0: the layer has none */
  int tied_values;          /* rotary: the values are the keys before rotation (vdim = dim) */
  int q_rank, kv_rank;      /* latent: sizes of the query's and of the key / value latent */
  int rot_part;             /* latent: size of the rotated part of q and k, behind the `dim` unrotated ones of a head */
  int head_gate;            /* latent: a head's output is multiplied by sigmoid of its row of in_proj */
  int experts, top;         /* 0: PolyNorm feed-forward; else a mixture of that many experts, `top` of them per token */
  float expert_limit;
} w4a32_layer_config;

typedef struct {
  int hidden, vocab, n_layers;
  int canon_taps;           /* taps of the input convolution of both sublayers (0: none, with W4A32_NORM_RMS) */
  float norm_eps;
  int dtype;                /* W4A32_LAYERED_* */
  int max_seq;              /* tokens a sequence's caches hold */
  int max_batch_tokens;     /* most tokens one call takes */
  const w4a32_layer_config* layers; /* HOST array */
  int norm;                 /* W4A32_NORM_* */
  float residual_mult;      /* factor of what a sublayer adds to the residual stream; 0 stands for 1 */
  int loop_start, loop_stop, loop_times; /* loop_times 0: no loop */
} w4a32_layered_config;

/* Device pointers. Rows of in_proj, all in one matrix, in this order:
 *   attention  q [heads*dim], k [kv_heads*dim], v [kv_heads*vdim]         (kv_from >= 0: q only)
 *   delta      q [kv_heads*dim], k [kv_heads*dim], v [heads*vdim], gate [heads*vdim], a [heads], b [heads]
 *   retention  q [heads*dim], k [heads*dim], v [heads*vdim], gate [heads*vdim]
 *   rotary     q [heads*dim], k [kv_heads*dim], v [kv_heads*vdim] (tied_values: no v)
 *   latent     query latent [q_rank], key / value latent [kv_rank], key part [rot_part], gate [heads] (head_gate)
 * conv: the short convolution's weights over the q, k, v rows in the same order, transposed: [taps][pad(rows)].
 * Operand blocks: k_up and v_up hold w4a32_layered_head_rows() rows per head (the true ones first, then zeros) and
 * pad(kv_rank) columns, element (row r, column c) at (((r / 32) * (pad(kv_rank) / 8) + c / 8) * 32 + r % 32) * 8 + c % 8.
 * gate_up: per expert 2 pad(ff) rows in groups of 64: 32 rows of gate, then the same 32 rows of up. */
typedef struct {
  const float *norm1, *norm2;      /* [pad(hidden)] */
  const float *canon1, *canon2;    /* [canon_taps][pad(hidden)] */
  const void* in_proj;             /* T [pad(rows)][pad(hidden)] */
  const float* conv;
  const void* out_proj;            /* T [pad(hidden)][pad(heads*vdim)] */
  const float *a_log, *dt_bias;    /* delta: [heads] */
  const float* head_norm;          /* delta: [vdim] */
  const float *decay, *log_decay;  /* retention: [heads], the decay and its natural logarithm */
  const void* up;                  /* T [pad(ff)][pad(hidden)] */
  const void* down;                /* T [pad(hidden)][pad(ff)] */
  const float* act;                /* PolyNorm a, b, c, e */
  const float* sinks;              /* rotary, latent: [heads], or null */
  const float *q_norm, *kv_norm;   /* latent: [pad(q_rank)], [pad(kv_rank)] */
  const void* q_up;                /* latent: T [pad(heads*(dim+rot_part))][pad(q_rank)], head by head */
  const void *k_up, *v_up;         /* latent: T, operand blocks of heads*dim and heads*vdim rows */
  const void* router;              /* experts: T [pad(experts)][pad(hidden)] */
  const void* gate_up;             /* experts: T [experts][2 pad(ff)][pad(hidden)] */
  const void* experts_down;        /* experts: T [experts][pad(hidden)][pad(ff)] */
} w4a32_layered_layer;

typedef struct {
  const void* embedding;           /* T [vocab][pad(hidden)] */
  const float* final_norm;         /* [pad(hidden)] */
  const void* head;                /* T [vocab][pad(hidden)] */
  const w4a32_layered_layer* layers; /* HOST array */
  const void* loop_in;             /* T [pad(hidden)][2 pad(hidden)]: the columns of x, then those of the embedding row */
} w4a32_layered_weights;

/* W4A32_OK, or why the configuration cannot run: W4A32_EINVAL (a size out of range), W4A32_ESHAPE (sizes that do
 * not fit each other), W4A32_ENOTSUP (beyond the limits above, or a row too long for the LDS). */
int w4a32_layered_check(const w4a32_layered_config* cfg);

/* Rows per head of k_up and v_up for these head sizes. */
int w4a32_layered_head_rows(int dim, int vdim);
/* Layer runs of a pass through the model (a looped layer counts once per pass). */
int w4a32_layered_runs(const w4a32_layered_config* cfg);

/* What one sequence keeps (caches, convolution tails, recurrent states, position), and what a call works in
 * (activations, rotation tables; shared by all sequences of a model). 256-byte aligned bases. 0: see _check. */
size_t w4a32_layered_state_bytes(const w4a32_layered_config* cfg);
size_t w4a32_layered_workspace_bytes(const w4a32_layered_config* cfg);
/* Byte offset of the position counter (int32) in the state / of the residual stream rows (f32
 * [max_batch_tokens][pad(hidden)], as the last layer left them) in the workspace, for inspection. */
size_t w4a32_layered_position_offset(const w4a32_layered_config* cfg);
size_t w4a32_layered_residual_offset(const w4a32_layered_config* cfg);

/* Once per allocation: clears it (the caches' padding must be finite) and, in the workspace, builds the rotation
 * tables. A state that was used is ready for another sequence as it is: that sequence starts at position 0. */
int w4a32_layered_init_state(const w4a32_layered_config* cfg, void* d_state, void* stream);
int w4a32_layered_init_workspace(const w4a32_layered_config* cfg, void* d_ws, void* stream);

/* n_tokens tokens of a sequence at positions pos0 .. through the model, from the state earlier calls left (pos0 is
 * the number of tokens they ran). Logits of the rows d_want[0..n_want) (indices among these tokens, device memory)
 * go to d_logits [n_want][vocab]; n_want may be 0. stop_after > 0 stops behind that many layer runs and writes no
 * logits (the residual stream is left for inspection); 0: the whole model. */
int w4a32_layered_forward(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                          const int64_t* d_tokens, int n_tokens, int pos0, const int* d_want, int n_want,
                          float* d_logits, int stop_after, void* stream);

/* The same for a prompt slice, then the greedy choice after its last token -> *d_next_token (int64). */
int w4a32_layered_prefill(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                          const int64_t* d_tokens, int n_tokens, int pos0, int64_t* d_next_token, void* stream);

/* One greedy decode step at the state's current position: reads *d_token_in, writes *d_token_out (may be the same
 * address), advances the position. The launch sequence does not depend on the position (capture once, replay per
 * token). The caller keeps the position below max_seq; past it the step stays inside its memory and its token is
 * meaningless. */
int w4a32_layered_step(const w4a32_layered_config* cfg, const w4a32_layered_weights* w, void* d_state, void* d_ws,
                       const int64_t* d_token_in, int64_t* d_token_out, void* stream);

/* ---- operators --------------------------------------------------------------------------------- */

/* C[M][N] = A[M][K] B[N][K]^T, both bf16 with leading dimension K (K % 64 == 0), f32 accumulation. C is f32 (c_bf16
 * == 0) or bf16, leading dimension ldc. With parts > 1 the k range is dealt to that many groups of workgroups and C
 * receives [parts][M][ldc] f32 partial products. */
int w4a32_op_matmul_bf16_nt(const void* d_a, const void* d_b, void* d_c, int M, int N, int K, int ldc, int c_bf16,
                            int parts, void* stream);

/* x_out = x + sum of n_parts partial rows [n_parts][M][ld] (skipped when n_parts is 0; x_out must not alias x);
 * h = (x_out - mean) / sqrt(variance + eps) * w over the first H of ld = pad(H) channels; y = h + conv(h) with the
 * `taps` x [ld] weights d_conv (taps 0: y = h). Row m has position pos0 + m; d_ring [taps][ld] holds h of the last
 * positions (slot: position % taps) and is updated. y is bf16 or f32 [M][ld]. */
int w4a32_op_layernorm_conv(const float* d_x, const float* d_parts, int n_parts, float* d_x_out, const float* d_norm,
                            float eps, const float* d_conv, float* d_ring, int taps, int M, int H, int pos0,
                            void* d_y, int y_bf16, void* stream);

/* y = silu(conv(x)) (or conv(x)) per channel: x f32 [M][ldx], y f32 [M][ldy], weights [taps][ldw], ring [taps][ldw]
 * of x as above. */
int w4a32_op_short_conv(const float* d_x, int ldx, float* d_y, int ldy, const float* d_w, float* d_ring, int ldw,
                        int taps, int channels, int apply_silu, int M, int pos0, void* stream);

/* The rows' mixture of experts: h T [M][pad(hidden)], router logits f32 [M][ld] -> d_parts f32 [top][M][pad(hidden)], one
 * row per chosen expert, weighted. d_scratch: w4a32_op_experts_scratch_bytes bytes, 256-byte aligned. */
size_t w4a32_op_experts_scratch_bytes(int dtype, int M, int experts, int top, int ff);
int w4a32_op_experts(int dtype, const void* d_h, const float* d_logits, int ld, const void* d_gate_up, const void* d_down,
                     int M, int hidden, int experts, int top, int ff, float limit, float* d_parts, void* d_scratch,
                     void* stream);

/* In place: z [M][ld] bf16 or f32, F channels; z <- PolyNorm(z) with the four numbers at d_act. */
int w4a32_op_polynorm(void* d_z, int z_bf16, int M, int F, int ld, const float* d_act, float eps, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* W4A32_LAYERED_H */
