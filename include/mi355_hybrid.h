/* C ABI of the layer-list ("hybrid") host layer: decoder-only models whose config lists, layer by layer, which token mixer a
 * layer has -- sliding-window attention with a softmax sink, a gated delta rule (recurrent matrix state), a minGRU (recurrent vector
 * state), attention and delta rule side by side, latent attention (keys and values read off one cached latent vector per token), or
 * attention behind a short convolution whose heads' softmax weights are mixed -- and which feed-forward (dense gate/up forms or a
 * mixture of experts), a state-space mixer with a scalar decay per head, or linear attention with one constant decay per head; the
 * residual stream is one vector per token or several mixed copies of it; time mixing (projections of a token mixed with the one before,
 * a matrix state with a decay per key channel, a bonus for the current token).  The Sogodra, Vivazen, Kerolorn, Sabolorn, Tosivik and
 * Devalorn designs are its users.
 *
 * What differs from the llama-family host layers (mi355_llama_*, mi355_dense_*):
 *   - the residual stream, norms, attention scores, decays, gates of a recurrence and the recurrent state are f32 in both dtypes;
 *     `dtype` = MI355_DTYPE_BF16 keeps the matrices (and the K/V pages) in bf16 and multiplies on the matrix cores with f32
 *     accumulation, MI355_DTYPE_F32 keeps everything in f32 and multiplies with plain f32 FMAs (no reduced-precision mode);
 *   - one step function for prompts, portions of prompts and single decoded tokens: every sequence of a step brings
 *     cu_seqlens_q[i+1] - cu_seqlens_q[i] new tokens behind context_lens[i] - that many cached ones (the fields of
 *     mi355_be_prepare_prompt); K/V live in the block engine's pages, recurrent state in the block engine's state slots
 *     (mi355_be_state_*), one slot per live sequence;
 *   - a sequence whose portion starts at position 0 starts from zero state whatever its slot held before.
 * Every entry point returns 0 on success (hipError_t or a negative argument error otherwise) and only enqueues work on `stream`. */
#pragma once
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define MI355_HYB_MIX_PARALLEL 0   /* attention ("left") and gated delta rule ("right") on the same input, outputs scaled and added */
#define MI355_HYB_MIX_MINGRU 1
#define MI355_HYB_MIX_DELTA 2
#define MI355_HYB_MIX_ATTENTION 3  /* the attention branch alone */
#define MI355_HYB_MIX_LATENT 4     /* latent attention: the pages hold [latent c (a_kv_rank) | rotated key part (a_rot_dim)] per token;
                                      head h's key is W_uk,h c and its value W_uv,h c.  Computed in the absorbed form: the query
                                      carries W_uk,h^T q_h, the attention runs over the latent rows themselves (one shared key/value
                                      head of a_kv_rank + a_rot_dim / a_kv_rank dimensions), W_uv,h is applied to its output */
#define MI355_HYB_MIX_CONV_ATTENTION 5 /* q, k, v pass a short causal convolution (a_conv taps, no activation), then attention with
                                      the a_* switches below; the convolution's last inputs live in the state slot */

#define MI355_HYB_MIX_SSD 6         /* selective state-space mixer (scalar decay per head): the input projection gives [gate z | x | B | C |
                                      step dt]; x, B, C pass a short causal convolution with bias and silu; per head S <- exp(-exp(a_log)
                                      dt) S + dt B x^T, y = S^T C + skip x; y silu(z), RMS norm in d_norm_groups parts, output projection.
                                      d_heads heads of d_vdim, state size d_dim, d_kv_heads groups of B / C, d_conv taps            */

#define MI355_HYB_MIX_DECAY 7       /* linear attention with a constant decay per head: q, k, v = silu of their projections (d_heads heads of
                                      d_dim | d_vdim, no sharing), S <- decay[h] S + k v^T, o = S^T q; RMS norm over all heads together,
                                      times sigmoid(W_g h), output projection.  The decays are MI355_HW_D_DECAY                       */

#define MI355_HYB_MIX_TIMEMIX 8     /* time mixing: with h' the token before (zeros at the start), r, k, v, gate and decay input each read
                                      h + (h' - h) mu_s (MI355_HW_T_MU); log w = -exp(W_2 tanh(W_1 mix) + w_0) per head and key channel (rank
                                      d_a_rank); per head o = (S + diag(u) k v^T)^T r, then S <- diag(w) S + k v^T; o over its root mean square,
                                      times MI355_HW_D_NORM, times silu(gate), output projection.  d_heads heads of d_dim | d_vdim; the slot
                                      holds S and the last token's h.  Belongs to residual_form 5                                       */
#define MI355_HYB_MIX_PARALLEL_TIMEMIX 9 /* attention ("left") and time mixing ("right") on the same input, outputs scaled and added     */

#define MI355_HYB_MASK_SLIDING 0    /* a query at position i sees keys j with 0 <= i - j < window                                      */
#define MI355_HYB_MASK_CHUNKED 1    /* it sees keys j <= i with floor(i / window) = floor(j / window)                                  */

#define MI355_HYB_ACT_NONE 0        /* activations in the epilogue of a product                                                        */
#define MI355_HYB_ACT_SILU 1
#define MI355_HYB_ACT_GELU 2        /* the tanh form                                                                                   */
#define MI355_HYB_ACT_RELU2 3       /* relu(z)^2                                                                                       */

#define MI355_HYB_GATE_SILU 0      /* output gate silu(W_g h), full rank                */
#define MI355_HYB_GATE_SIGMOID_LR 1 /* output gate sigmoid(W_g2 (W_g1 h)), low rank     */

typedef struct mi355_hybrid_layer {
    int32_t mixer;                 /* MI355_HYB_MIX_*                                                              */
    /* attention branch */
    int32_t a_heads, a_kv_heads, a_dim, a_vdim;
    int32_t a_window;              /* 0 = none; else a query at position i sees keys j with 0 <= i - j < a_window  */
    int32_t a_rot_dims;            /* leading dimensions of a head that are rotated (rotate-half pairs), 0 = none  */
    int32_t a_has_sink;            /* the softmax denominator also holds exp(sink[head])                           */
    int32_t a_qk_norm;             /* RMS norm of every query / key head before the rotation                       */
    float a_scale, a_out_scale;
    /* delta-rule branch */
    int32_t d_heads, d_kv_heads, d_dim, d_vdim, d_conv;
    int32_t d_decay_channels;      /* 0: one decay per head (full-rank W_a [heads, width]);
                                      1: one per head and key channel (low rank W_a2 (W_a1 h), rank d_a_rank)      */
    int32_t d_a_rank;
    int32_t d_gate;                /* MI355_HYB_GATE_*                                                             */
    int32_t d_g_rank;
    float d_out_scale;
    /* minGRU */
    int32_t g_width;
    /* feed-forward: 0 = none, 1 = dense clamped gate/up with y = g sigmoid(act_alpha g) (u + 1),
                     2 = dense gate/up with y = gelu_tanh(g) u,
                     3 = mixture of experts with y = silu(g) u (fields below; the shared expert, when there is one, uses the dense
                         slots MI355_HW_MLP_GATE_UP / _DOWN with moe_shared_ff)                                       */
    int32_t mlp_kind, mlp_ff;
    float mlp_limit, mlp_alpha;
    /* more switches of the attention branch (all 0 = the plain form) */
    int32_t a_rot_interleaved;     /* rotated pairs are (2i, 2i + 1) instead of (i, i + a_rot_dims / 2)                   */
    int32_t a_kv_rank, a_rot_dim;  /* latent attention: latent size; rotated dimensions per query head = the shared key part
                                      (a_dim = the unrotated dimensions per head, a_rot_dims <= a_rot_dim of them turn)    */
    int32_t a_head_gate;           /* head h's output times sigmoid((W_g x)_h), W_g [heads, width] in the input projection */
    int32_t a_conv;                /* taps of the convolution behind q, k, v                                               */
    int32_t a_norm_whole;          /* a_qk_norm is ONE RMS norm over all of q (and of k), weights [heads * dim]            */
    int32_t a_v_unit;              /* every value head is divided by its root mean square before it is cached             */
    float a_softcap;               /* > 0: score <- cap tanh(score / cap)                                                  */
    int32_t a_talk;                /* weight_h <- sum_g talk[h, g] weight_g after the softmax; head h applies its mixed
                                      weights to the values of its own key/value head                                      */
    int32_t share_with;            /* 0: the layer has weights; n > 0: it runs on layer n - 1's weights (and rope tables) with
                                      pages and state of its own                                                           */
    /* switches of the plain attention mixers (MI355_HYB_MIX_ATTENTION / _PARALLEL), all 0 = the form above */
    int32_t a_keep_first;          /* with a window: keys at positions < a_keep_first stay visible to every later query     */
    int32_t a_norm_after_rot;      /* the RMS norm of q and k (a_qk_norm) is taken AFTER the rotation and has no weight     */
    int32_t a_head_temp;           /* head h's scores are multiplied by temp[h] (MI355_HW_A_TEMP)                           */
    /* input convolution in front of the mixer: what the mixer reads, h, becomes h + conv(h), a causal convolution over time on
     * every channel of the width (in_conv taps, 0 = none); the last taps - 1 rows of h live in the state slot                  */
    int32_t in_conv;
    /* feed-forward kind 3, a mixture of experts: moe_experts gate/up experts of mlp_ff with silu, every token uses the moe_top with
     * the largest softmax(router) + correction; its weights are the chosen experts' softmax values times moe_scale (not
     * renormalised).  moe_shared_ff > 0: one more expert of that size runs for every token, times sigmoid(w_sg . h)              */
    int32_t moe_experts, moe_top, moe_shared_ff;
    float moe_scale;
    /* more switches of the router (all 0 = the form above) */
    int32_t moe_sigmoid;           /* scores are sigmoid(z) instead of softmax(z)                                           */
    int32_t moe_groups, moe_keep_groups; /* > 0: the experts form moe_groups equal groups of neighbours; a group's score is the sum of
                                      its two largest choice scores and only experts of the best moe_keep_groups groups can be chosen */
    int32_t moe_normalise;         /* the chosen experts' scores are divided by their sum (+ 1e-20) before moe_scale         */
    /* feed-forward kind 4: dense without a gate, y = W_down relu(W_up h)^2 (MI355_HW_MLP_GATE_UP holds the [ff, width] up rows)  */
    int32_t d_norm_groups;         /* MI355_HYB_MIX_SSD: parts of the gated output with a root mean square of their own      */
    int32_t a_dist_bias;           /* MI355_HYB_MIX_CONV_ATTENTION: score <- score - r1[h] ln(1 + r2[h] (i - j)), MI355_HW_A_DIST */
    int32_t a_q_rank;              /* latent attention, > 0: queries through a latent, q = W_uq RMSnorm(W_dq h) (MI355_HW_L_UQ,
                                      MI355_HW_L_QNORM); the q part of the input projection then holds the a_q_rank rows of W_dq */
    int32_t a_out_gate;            /* latent attention: the concatenated heads times sigmoid(W_g h) element by element, W_g
                                      [heads vdim, width] in the gate part of the input projection                            */
    int32_t kv_from;               /* latent attention, n > 0: no down-projection and no pages of its own; the layer reads the pages
                                      that layer n - 1 (an earlier latent layer of the same kv_rank / rot_dim) has written       */
    int32_t side_dim;              /* > 0: after the sublayers x <- x + RMSnorm(W_proj (gelu_tanh(W_gate x) * e)) w with e = the
                                      token's row of the side table, columns [side_col, side_col + side_dim)                   */
    int32_t side_col;
    int32_t depth_terms;           /* n > 0: behind the layer x <- sum_j w[j] X_j over the n earliest of (embedding output, results
                                      of the layers so far); n = layer index + 2 (MI355_HW_DEPTH_W [n])                        */
    /* more switches of the plain attention mixers */
    int32_t a_mask_kind;           /* MI355_HYB_MASK_*: what a_window means                                                  */
    int32_t a_v_is_k;              /* no value projection: the cached value row is the key as projected, before the rotation
                                      (a_vdim == a_dim); the v part of the input projection is its k part                    */
    /* more forms of the feed-forward.  mlp_kind 5: dense without a gate, y = W_down gelu_tanh(W_up h) (up rows as in kind 4) */
    int32_t moe_relu2;             /* kind 3: the experts (and the shared one) are y = W_down relu(W_up h)^2 without a gate; the
                                      GATE_UP slots then hold [ff, width] up rows per expert                                 */
    int32_t moe_bias;              /* kind 3: z = router . h + bias (MI355_HW_MOE_BIAS), softmax over the chosen logits only   */
    int32_t moe_shared_plain;      /* kind 3: the shared expert is added as it is (no gate row in the router)                  */
    /* more forms of the plain attention mixers: a_norm_whole (no rotation then), a_head_gate, a_softcap, kv_from (the lender: an earlier
     * layer with the same kv heads and head sizes; its keys as cached and its values), a_dist_bias 1 as above or 2: score <- score -
     * r1[h] (i - j) (MI355_HW_A_DIST as above, r2 unused).  mlp_kind 6: dense gate/up with y = silu(g) u (residual_form 5)       */
    float a_temp_coef, a_temp_every; /* != 0: the query at position p is multiplied by 1 + coef ln(floor((p + 1) / every) + 1)    */
} mi355_hybrid_layer;

typedef struct mi355_hybrid_config {
    int32_t width, vocab, n_layers;
    int32_t dtype;                 /* MI355_DTYPE_F32 or MI355_DTYPE_BF16                                          */
    int32_t block_size;            /* tokens per K/V page                                                          */
    int32_t state_slots;           /* recurrent-state slots (live sequences)                                       */
    float norm_eps;
    float unit_eps;                /* eps inside the root of the unit norm of q and k in the delta rule            */
    int32_t residual_form;         /* 0: x <- x + norm(sub(x));  1: x <- norm(resid_alpha x + sub(x));
                                      2: x <- x + norm(sub(pre_norm(x))), a norm on both sides of every sublayer
                                         (MI355_HW_PRE_NORM1 / 2 in front, MI355_HW_NORM1 / 2 behind)                 */
    float resid_alpha;
    int32_t norm_groups;           /* the layer norms and the last norm take the RMS over this many equal consecutive parts
                                      of the vector separately (0 or 1: over the whole vector)                       */
    float logit_scale;             /* the logits are multiplied by it (0 = 1)                                        */
    /* residual_form 3: ONE norm per layer, h = norm(x) (MI355_HW_NORM1), and both sublayers read it: x <- x + mixer(h) + ff(h) */
    int32_t norm_kind;             /* 0: RMS norm; 1: layer norm with a weight and no bias, (x - mean) / sqrt(var + eps) w -- the
                                      norm in front of the sublayers (form 3) and the last norm                              */
    float embed_scale;             /* the embedding rows are multiplied by it (0 = 1)                                        */
    float logit_softcap;           /* > 0: logits <- cap tanh(logits / cap)                                                  */
    int32_t tie_head;              /* the logits are taken against the embedding table itself; MI355_HW_HEAD stays empty     */
    int32_t side_cols;             /* columns of the per-layer token table MI355_HW_SIDE_TABLE [vocab, side_cols] (0 = none) */
    /* residual_form 4: the residual stream is `streams` copies X_i of the embedding output.  Every sublayer (norm in front:
     * MI355_HW_NORM1 / 2) reads one mixture of them and writes to all: y = sub(norm(sum_i in[i] X_i)),
     * X_j <- sum_i mix[i, j] X_i + out[j] y (MI355_HW_HC1_* in the mixer, _HC2_* in the feed-forward); the model's output is
     * the sum of the copies                                                                                                  */
    /* residual_form 5: x <- x + (mixer(norm1(x)) + ff(norm2(x))), both norms (MI355_HW_NORM1 / 2) of the same x                 */
    int32_t streams;
    int32_t bigram_buckets;        /* > 0: the embedding also takes row (previous token mul_prev + token mul_cur) mod buckets of
                                      MI355_HW_BIGRAM (row `buckets` at a sequence's first token); the previous token lives in
                                      the state slot                                                                          */
    int64_t bigram_mul_prev, bigram_mul_cur;
} mi355_hybrid_config;

/* weight slots: `layer` = -1 for the three global ones */
#define MI355_HW_EMBED 0           /* [vocab, width]                                                                */
#define MI355_HW_FINAL_NORM 1      /* [width]                                                                       */
#define MI355_HW_HEAD 2            /* [vocab, width]                                                                */
#define MI355_HW_NORM1 3           /* [width]  norm on the mixer's output                                           */
#define MI355_HW_NORM2 4           /* [width]  norm on the feed-forward's output                                    */
#define MI355_HW_IN_PROJ 5         /* every projection that reads the mixer's input, concatenated along the rows in
                                      the order of mi355_hybrid_in_proj_rows: [rows, width]                         */
#define MI355_HW_IN_BIAS 6         /* [rows] or absent                                                              */
#define MI355_HW_OUT_PROJ 7        /* [width, k]: the output projections side by side along k (attention first)     */
#define MI355_HW_A_QNORM 8
#define MI355_HW_A_KNORM 9
#define MI355_HW_A_SINK 10
#define MI355_HW_D_CONV 11         /* [q channels + k channels + v channels, taps], last column = the current token */
#define MI355_HW_D_A_LOG 12        /* [heads]                                                                       */
#define MI355_HW_D_DT_BIAS 13      /* [heads] or [heads * dim]                                                      */
#define MI355_HW_D_NORM 14         /* [vdim]                                                                        */
#define MI355_HW_D_A2 15           /* [heads * dim, a_rank]                                                         */
#define MI355_HW_D_G2 16           /* [heads * vdim, g_rank]                                                        */
#define MI355_HW_MLP_GATE_UP 17    /* [2 ff, width]: gate rows, then up rows                                        */
#define MI355_HW_MLP_DOWN 18       /* [width, ff]                                                                   */
#define MI355_HW_A_CONV 19         /* [q channels + k channels + v channels, taps], last column = the current token */
#define MI355_HW_A_TALK 20         /* [heads, heads]                                                                */
#define MI355_HW_L_UKT 21          /* [heads, kv_rank, dim]: per head the TRANSPOSE of its block of W_uk [heads dim, kv_rank] */
#define MI355_HW_L_UV 22           /* [heads vdim, kv_rank]                                                         */
#define MI355_HW_L_CNORM 23        /* [kv_rank] weight of the latent's RMS norm                                      */
#define MI355_HW_PRE_NORM1 24      /* [width]  residual form 2: norm in front of the mixer                           */
#define MI355_HW_PRE_NORM2 25      /* [width]  residual form 2: norm in front of the feed-forward                    */
#define MI355_HW_IN_CONV 26        /* [width, in_conv], last column = the current token                              */
#define MI355_HW_A_TEMP 27         /* [heads]                                                                        */
#define MI355_HW_MOE_ROUTER 28     /* f32 [experts (+ 1 when moe_shared_ff: the shared expert's gate row last), width] */
#define MI355_HW_MOE_CORRECTION 29 /* [experts] added to the softmax values for the choice only                      */
#define MI355_HW_MOE_GATE_UP 30    /* [experts, 2 ff, width]: per expert gate rows, then up rows; a shared expert of the
                                      experts' size (moe_shared_ff == mlp_ff) is one more matrix at the end, here and in
                                      MOE_DOWN, and the dense slots stay empty                                       */
#define MI355_HW_MOE_DOWN 31       /* [experts, width, ff]                                                           */
#define MI355_HW_D_SKIP 32         /* [heads]  state-space mixer: y += skip[h] x                                     */
#define MI355_HW_CONV_BIAS 33      /* [channels] bias of the convolution MI355_HW_D_CONV                             */
#define MI355_HW_A_DIST 34         /* [2, heads]: r1, then r2 of the distance bias                                   */
#define MI355_HW_L_QNORM 35        /* [q_rank] weight of the query latent's RMS norm                                 */
#define MI355_HW_L_UQ 36           /* [heads (dim + rot_dim), q_rank]                                                */
#define MI355_HW_SIDE_GATE 37      /* [side_dim, width]                                                              */
#define MI355_HW_SIDE_PROJ 38      /* [width, side_dim]                                                              */
#define MI355_HW_SIDE_NORM 39      /* [width]                                                                        */
#define MI355_HW_DEPTH_W 40        /* [depth_terms]                                                                  */
#define MI355_HW_SIDE_TABLE 41     /* global (layer -1): [vocab, side_cols]                                          */
#define MI355_HW_HC1_IN 42         /* [streams]          residual form 4, mixer: what it reads of every copy         */
#define MI355_HW_HC1_OUT 43        /* [streams]          how much of its output every copy takes                     */
#define MI355_HW_HC1_MIX 44        /* [streams, streams] from copy i (row) to copy j                                 */
#define MI355_HW_HC2_IN 45         /* the same three of the feed-forward                                             */
#define MI355_HW_HC2_OUT 46
#define MI355_HW_HC2_MIX 47
#define MI355_HW_MOE_BIAS 48       /* [experts]                                                                      */
#define MI355_HW_D_DECAY 49        /* [heads] f32, mi355_hybrid_set_weight_f32                                       */
#define MI355_HW_BIGRAM 50         /* global (layer -1): [bigram_buckets + 1, width]                                 */
#define MI355_HW_T_MU 51           /* [5, width]  time mixing: the mixtures of r, k, v, gate, decay                  */
#define MI355_HW_T_W2 52           /* [d_a_rank, heads * dim]: the TRANSPOSE of W_2                                   */
#define MI355_HW_T_W0 53           /* [heads * dim]                                                                  */
#define MI355_HW_T_BONUS 54        /* [heads * dim]                                                                  */
#define MI355_HW_COUNT 55

void* mi355_hybrid_create(const mi355_hybrid_config* cfg, const mi355_hybrid_layer* layers);
void mi355_hybrid_destroy(void* model);
/* rows of a layer's concatenated input projection, and where each part starts: parts = attention q, k, v, delta q, k, v, beta,
 * decay (a or a1), gate (g or g1) for the attention / delta / parallel mixers; z, x, g for the minGRU; q (heads x (dim + rot_dim)),
 * the latent down-projection (kv_rank + rot_dim) in the k part and the head gate in the gate part for latent attention.  Time mixing: r, k, v
 * in the delta q, k, v parts, its gate in the beta part, W_1 in the decay part; the attention's rows together and every one of these
 * parts are followed by rows of zeros up to a multiple of 128 (the attention's head gate, where there is one, is in the gate part).
 * offsets[9], -1 = absent */
int32_t mi355_hybrid_in_proj_rows(const mi355_hybrid_layer* layer, int32_t* offsets);
/* HOST bf16 bits (a checkpoint tensor), n elements; converted to the storage type of the slot */
int mi355_hybrid_set_weight(void* model, int32_t layer, int32_t which, const uint16_t* host_bf16, int64_t n);
/* HOST f32 values of a slot that is kept in f32 (constants of a configuration that bf16 cannot hold) */
int mi355_hybrid_set_weight_f32(void* model, int32_t layer, int32_t which, const float* host, int64_t n);
/* DEVICE bf16 bits (synthetic weights of a benchmark) */
int mi355_hybrid_set_weight_dev(void* model, int32_t layer, int32_t which, const uint16_t* dev_bf16, int64_t n, int64_t stream);
/* HOST f32 [n_positions, a_rot_dims / 2] cos and sin of a layer's rotary angles (mi355_rope_tables builds them) */
int mi355_hybrid_set_rope_tables(void* model, int32_t layer, const float* cos_t, const float* sin_t, int32_t n_positions);
/* K/V pages of every attention layer and the state pool; all state starts as zero */
int mi355_hybrid_alloc_cache(void* model, int32_t num_blocks);
int64_t mi355_hybrid_cache_bytes(void* model, int32_t num_blocks);
int64_t mi355_hybrid_state_floats_per_slot(void* model);
void* mi355_hybrid_state_ptr(void* model);
/* one step over DEVICE inputs.  tokens u32 [T]; positions, slot_mapping i64 [T]; block_tables u32 [num_seqs, max_blocks];
 * context_lens u32 [num_seqs] (cached + new); cu_seqlens_q u32 [num_seqs + 1]; state_slots i32 [num_seqs]; out_rows i32 [n_out]
 * = the token rows whose logits are wanted -> logits f32 [n_out, vocab].  layer_trace: NULL, or f32 [n_layers, T, width] that
 * receives the residual stream behind every layer (parity hook). */
int mi355_hybrid_forward(void* model, const uint32_t* tokens, const int64_t* positions, const int64_t* slot_mapping,
                         const uint32_t* block_tables, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                         const int32_t* state_slots, const int32_t* out_rows, int32_t n_out, int32_t num_seqs, int32_t num_tokens,
                         int32_t max_blocks, int32_t max_context_len, float* logits, float* layer_trace, int64_t stream);

/* the same step from a hipGraph keyed by the device pointers and the counts (the caller keeps its step inputs in static device
 * buffers); `stream` must not be the default stream; no layer trace */
int mi355_hybrid_forward_graph(void* model, const uint32_t* tokens, const int64_t* positions, const int64_t* slot_mapping,
                               const uint32_t* block_tables, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                               const int32_t* state_slots, const int32_t* out_rows, int32_t n_out, int32_t num_seqs,
                               int32_t num_tokens, int32_t max_blocks, int32_t max_context_len, float* logits, int64_t stream);
int64_t mi355_hybrid_graph_captures(void* model);
int64_t mi355_hybrid_graph_replays(void* model);

/* ---- the mechanisms alone (tests, other host layers).  `dtype` is the type of 16/32-bit operands marked (dt); the rest is f32 */
/* token_seq i32 [T]: the sequence (row of cu_seqlens_q) of every token row */
int mi355_hyb_token_seq(int32_t* token_seq, const uint32_t* cu_seqlens_q, int32_t num_seqs, int64_t stream);
int mi355_hyb_bf16_to_f32(float* out, const uint16_t* in, int64_t n, int64_t stream);
int mi355_hyb_copy_f32(float* out, const float* in, int64_t n, int64_t stream);
int mi355_hyb_fill_f32(float* out, float v, int64_t n, int64_t stream);
/* x f32 [T, width] = table (dt) [vocab, width] rows ids; xcopy: NULL or bf16 [T, width] */
int mi355_hyb_embed(float* x, void* xcopy, const void* table, const uint32_t* ids, int32_t num_tokens, int32_t width, int32_t vocab,
                    int32_t dtype, int64_t stream);
/* out (dt_out) [n_rows, width] = RMS norm with weight of the rows `rows` of x */
int mi355_hyb_gather_norm(void* out, int32_t out_dtype, const float* x, const int32_t* rows, const float* w, int32_t n_rows,
                          int32_t width, float eps, int64_t stream);
/* out f32 [T, ldo] = a (dt_a: F32 or BF16) [T, lda] . w (dt) [n, k]^T + bias f32 [n] */
int mi355_hyb_linear(float* out, int32_t ldo, const void* a, int32_t a_dtype, int32_t lda, const void* w, const float* bias,
                     int32_t num_tokens, int32_t n, int32_t k, int32_t dtype, int64_t stream);
/* x f32 [T, width] += y / rms(y) * w, y f32 [T, ldy]; xcopy (NULL or bf16 [T, width]) receives the rounded sum */
int mi355_hyb_norm_add(float* x, void* xcopy, const float* y, int32_t ldy, const float* w, int32_t num_tokens, int32_t width,
                       float eps, int64_t stream);
/* per-head RMS norm (weights NULL = none) and rotation of q / k out of the projection rows, q -> q_out (dt) [T, heads, dim],
 * k, v -> the pages at slot_mapping (dt), [blocks, block_size, kv_heads, dim | vdim] */
int mi355_hyb_attn_prepare(void* q_out, void* k_pages, void* v_pages, const float* proj, int32_t ldp, int32_t q_off, int32_t k_off,
                           int32_t v_off, const float* q_norm_w, const float* k_norm_w, const float* cos_t, const float* sin_t,
                           const int64_t* positions, const int64_t* slot_mapping, int32_t num_tokens, int32_t heads,
                           int32_t kv_heads, int32_t dim, int32_t vdim, int32_t rot_dims, float eps, int32_t dtype, int64_t stream);
/* causal attention of every new token over its sequence's pages: window (0 = none), sink f32 [heads] or NULL;
 * out (dt_out) [T, ldo] at column out_off: heads x vdim, times out_scale */
int mi355_hyb_window_attention(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages,
                               const void* v_pages, const uint32_t* block_tables, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* token_seq, const float* sink, int32_t num_seqs, int32_t num_tokens,
                               int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size, int32_t max_blocks,
                               int32_t window, float scale, float out_scale, int32_t dtype, int64_t stream);
/* the same with the remaining switches: k_ld / v_ld = elements per page row of the key / value pages (0: kv_heads x dim | vdim;
 * latent attention passes the same pages for both with v_ld = k_ld), softcap (0 = none), cross_values: 1 = every query head's
 * weights are applied to the values of EVERY key/value head c, out [T, heads, kv_heads, vdim] (what mi355_hyb_head_mix reads) */
int mi355_hyb_window_attention_ex(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages,
                                  const void* v_pages, const uint32_t* block_tables, const uint32_t* context_lens,
                                  const uint32_t* cu_seqlens_q, const int32_t* token_seq, const float* sink, int32_t num_seqs,
                                  int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size,
                                  int32_t max_blocks, int32_t window, float scale, float out_scale, int32_t k_ld, int32_t v_ld,
                                  float softcap, int32_t cross_values, int32_t dtype, int64_t stream);
/* out (dt_out) [T, heads x vdim] = sum_g talk[h, g] a[t, g, kv head of h, :],  a f32 [T, heads, kv_heads, vdim]: mixing the heads'
 * softmax weights before the value product is the same as mixing, per key/value head, the outputs the unmixed weights give */
int mi355_hyb_head_mix(void* out, int32_t out_dtype, const float* a, const float* talk, int32_t num_tokens, int32_t heads,
                       int32_t kv_heads, int32_t vdim, int64_t stream);
/* out (dt_out) [T, heads x vdim] = in f32 [T, heads x vdim] times sigmoid(gate_in[t, h]) per head (gate_in NULL: a plain copy) */
int mi355_hyb_head_gate(void* out, int32_t out_dtype, const float* in, const float* gate_in, int32_t ldg, int32_t num_tokens,
                        int32_t heads, int32_t vdim, int64_t stream);
/* attention behind a convolution: src f32 [T, ld] holds q | k | v rows (offsets q_off, k_off, v_off).  q and k: RMS norm over the WHOLE
 * row part (heads x dim, kv_heads x dim) with weights of that size (NULL = no norm); v: every head divided by its root mean square when
 * v_unit.  q -> q_out (dt) [T, heads, dim], k, v -> the pages at slot_mapping.  No rotation */
int mi355_hyb_attn_prepare_whole(void* q_out, void* k_pages, void* v_pages, const float* src, int32_t ld, int32_t q_off, int32_t k_off,
                                 int32_t v_off, const float* q_norm_w, const float* k_norm_w, const int64_t* slot_mapping,
                                 int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t v_unit, float eps,
                                 int32_t dtype, int64_t stream);
/* latent attention: proj f32 [T, ldp] holds per head [dim unrotated | rot_dim rotated] query rows at q_off and the down-projection
 * [kv_rank | rot_dim] at c_off; q_abs f32 [T, heads, kv_rank] = the unrotated query parts already multiplied by W_uk^T.
 * pages (dt) [.., kv_rank + rot_dim] at slot_mapping <- [RMS norm of the latent times c_norm_w | rotated key part];
 * q_out (dt) [T, heads, kv_rank + rot_dim] <- [q_abs | rotated query part].  The first rot_dims of the rot_dim dimensions turn
 * (pairs (2i, 2i+1) when interleaved), cos_t / sin_t [positions, rot_dims / 2] carry any amplitude */
int mi355_hyb_latent_prepare(void* q_out, void* pages, const float* proj, int32_t ldp, int32_t q_off, int32_t c_off, const float* q_abs,
                             const float* c_norm_w, const float* cos_t, const float* sin_t, const int64_t* positions,
                             const int64_t* slot_mapping, int32_t num_tokens, int32_t heads, int32_t dim, int32_t rot_dim,
                             int32_t kv_rank, int32_t rot_dims, int32_t interleaved, float eps, int32_t dtype, int64_t stream);
/* `batch` independent products of one shape in one launch: out + z o_bs [T, ldo] = (a + z a_bs) [T, lda] . (w + z w_bs) [n, k]^T,
 * strides in elements (per-head matrices: z = head) */
int mi355_hyb_linear_batched(float* out, int32_t ldo, int64_t o_bs, const void* a, int32_t a_dtype, int32_t lda, int64_t a_bs,
                             const void* w, int64_t w_bs, int32_t num_tokens, int32_t n, int32_t k, int32_t batch, int32_t dtype,
                             int64_t stream);
/* x f32 [T, width] <- group norm(alpha x + y) times w (the norm BEHIND the residual sum; `groups` equal consecutive parts, each with
 * its own root mean square); xcopy: NULL or bf16 [T, width] */
int mi355_hyb_resid_norm(float* x, void* xcopy, const float* y, int32_t ldy, const float* w, int32_t num_tokens, int32_t width,
                         int32_t groups, float alpha, float eps, int64_t stream);
/* mi355_hyb_gather_norm with the RMS taken over `groups` parts */
int mi355_hyb_gather_group_norm(void* out, int32_t out_dtype, const float* x, const int32_t* rows, const float* w, int32_t n_rows,
                                int32_t width, int32_t groups, float eps, int64_t stream);
/* out (dt_out) [T, ff] = gelu_tanh(gu[:, j]) gu[:, ff + j] */
int mi355_hyb_gelu_glu(void* out, int32_t out_dtype, const float* gu, int32_t num_tokens, int32_t ff, int64_t stream);
/* mi355_hyb_conv_silu with the activation as an argument: 0 = none, 1 = silu */
int mi355_hyb_conv(float* out, const float* proj, int32_t ldp, int32_t off, const float* w, const float* conv_state,
                   int64_t state_stride, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                   const int32_t* token_seq, int32_t num_seqs, int32_t num_tokens, int32_t channels, int32_t taps, int32_t act,
                   int64_t stream);
/* ---- mechanisms of the pre/post-norm designs */
/* out (dt_out) [T, width] = RMS norm of every row of x times w (the norm in front of a sublayer) */
int mi355_hyb_pre_norm(void* out, int32_t out_dtype, const float* x, const float* w, int32_t num_tokens, int32_t width, float eps,
                       int64_t stream);
/* out (dt_out) [T, channels] = h + conv(h) for h = in f32 [T, ld] columns [off, off + channels): the causal convolution of
 * mi355_hyb_conv added to its own input; mi355_hyb_conv_state_update(in) then moves the state behind the portion */
int mi355_hyb_conv_residual(void* out, int32_t out_dtype, const float* in, int32_t ld, int32_t off, const float* w,
                            const float* conv_state, int64_t state_stride, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                            const int32_t* state_slots, const int32_t* token_seq, int32_t num_seqs, int32_t num_tokens, int32_t channels,
                            int32_t taps, int64_t stream);
/* the two above in ONE launch for taps <= 8: h = RMS norm of x times norm_w (norm_w NULL: h = x), out (dt_out) [T, width] = h + conv(h).
 * hn: NULL, or f32 [T, width] that receives h (what mi355_hyb_conv_state_update then reads).  update_state != 0 (only when every
 * sequence brings one token, T == num_seqs): the kernel moves the state behind the token itself and no update launch is needed */
int mi355_hyb_norm_conv(void* out, int32_t out_dtype, float* hn, const float* x, const float* norm_w, const float* conv_w, float* conv_state,
                        int64_t state_stride, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                        const int32_t* token_seq, int32_t num_seqs, int32_t num_tokens, int32_t width, int32_t taps, int32_t update_state,
                        float eps, int64_t stream);
/* mi355_hyb_attn_prepare with the remaining switches: interleaved = rotated pairs are (2i, 2i + 1); norm_mode 0 = none, 1 = RMS norm
 * with weights before the rotation (q_norm_w / k_norm_w, NULL = no weight), 2 = RMS norm without a weight AFTER the rotation;
 * q_head_scale f32 [heads] or NULL: head h's query is multiplied by it (a temperature per head folded into the query) */
int mi355_hyb_attn_prepare_ex(void* q_out, void* k_pages, void* v_pages, const float* proj, int32_t ldp, int32_t q_off, int32_t k_off,
                              int32_t v_off, const float* q_norm_w, const float* k_norm_w, const float* cos_t, const float* sin_t,
                              const int64_t* positions, const int64_t* slot_mapping, int32_t num_tokens, int32_t heads,
                              int32_t kv_heads, int32_t dim, int32_t vdim, int32_t rot_dims, int32_t interleaved, int32_t norm_mode,
                              const float* q_head_scale, float eps, int32_t dtype, int64_t stream);
/* mi355_hyb_window_attention_ex with kept first tokens: beside the keys inside its window (all earlier keys when window == 0) a query
 * sees the keys at positions below keep_first; those keep their own positions and rotations */
int mi355_hyb_masked_attention(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages,
                               const void* v_pages, const uint32_t* block_tables, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* token_seq, const float* sink, int32_t num_seqs,
                               int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size,
                               int32_t max_blocks, int32_t window, int32_t keep_first, float scale, float out_scale, int32_t k_ld,
                               int32_t v_ld, float softcap, int32_t cross_values, int32_t dtype, int64_t stream);
/* mixture of experts, routing: h = RMS norm of x times norm_w (norm_w NULL: h = x) -> xn (dt_out) [T, width] (NULL = not written);
 * z = router f32 [experts, width] . h in f32, s = softmax(z); the `top` experts with the largest s + correction (correction NULL =
 * none; ties to the lower expert) -> expert_ids i32 [T, top] in descending order of the choice score, weights f32 [T, top] =
 * s[chosen] * scale.  gate_row f32 [width] or NULL: shared_gate f32 [T] (NULL = not written) = sigmoid(gate_row . h).
 * append_shared: expert_ids and weights are [T, top + 1] and every token's last pair is (expert `experts`, that sigmoid): a shared
 * expert of the experts' size runs as one more group of the grouped products */
int mi355_hyb_moe_route(int32_t* expert_ids, float* weights, float* shared_gate, void* xn, int32_t out_dtype, const float* x,
                        const float* norm_w, const float* router, const float* correction, const float* gate_row, int32_t num_tokens,
                        int32_t width, int32_t experts, int32_t top, float scale, float eps, int32_t append_shared, int64_t stream);
/* rows of a grouped product's blocks that suit `pairs` (token, expert) pairs over `experts` experts with [n, k] matrices: 16 (few
 * rows per expert: a stream over the weights), 64 or 128 (matrix-core tiles through LDS) */
int32_t mi355_hyb_moe_block_rows(int32_t pairs, int32_t experts, int32_t n, int32_t k, int32_t dtype);
/* grouping on the device: every expert owns whole blocks of block_rows rows of the gathered buffers, expert e's rows start at
 * block_rows * (blocks of the experts before it).  pos i32 [pairs] = the row of pair p = token * top + slot; row_token i32 [n_blocks *
 * block_rows] = the token of every used row; block_table i32 [n_blocks, 2] = {expert, one past the expert's last row} for every block
 * ({0, 0} past the last expert's), n_blocks >= ceil(pairs / block_rows) + experts */
int mi355_hyb_moe_group(int32_t* pos, int32_t* row_token, int32_t* block_table, const int32_t* expert_ids, int32_t pairs, int32_t top,
                        int32_t experts, int32_t block_rows, int32_t n_blocks, int64_t stream);
/* one product per block of the table: out f32 rows [b block_rows, block end) = a rows . (w + expert w_bs) [n, k]^T; a (dt_a) [.., lda]
 * row r is read at row_token[r] when row_token != NULL (gathered from the token rows), else at r */
int mi355_hyb_linear_grouped(float* out, int32_t ldo, const void* a, int32_t a_dtype, int32_t lda, const int32_t* row_token,
                             const void* w, int64_t w_bs, const int32_t* block_table, int32_t block_rows, int32_t n_blocks, int32_t n,
                             int32_t k, int32_t dtype, int64_t stream);
/* out (dt_out) [rows, ff] = silu(gu[:, j]) gu[:, ff + j]; block_table != NULL: only the rows that a block of the table uses */
int mi355_hyb_silu_glu(void* out, int32_t out_dtype, const float* gu, int32_t rows, int32_t ff, const int32_t* block_table,
                       int32_t block_rows, int64_t stream);
/* x f32 [T, width] += y / rms(y) * w with y[t] = sum_j weights[t, j] y_rows[pos[t top + j]] + shared_gate[t] y_shared[t]
 * (y_shared NULL = no shared expert; shared_gate NULL = 1); xcopy: NULL or bf16 [T, width] */
int mi355_hyb_moe_combine_norm_add(float* x, void* xcopy, const float* y_rows, const int32_t* pos, const float* weights,
                                   const float* y_shared, const float* shared_gate, const float* w, int32_t num_tokens, int32_t width,
                                   int32_t top, float eps, int64_t stream);
int mi355_hyb_scale_f32(float* x, float s, int64_t n, int64_t stream);
/* ---- mechanisms of the parallel-residual designs (hybrid_blocks.hip) */
/* x f32 [T, width] = table rows ids times scale */
int mi355_hyb_embed_scaled(float* x, const void* table, const uint32_t* ids, int32_t num_tokens, int32_t width, int32_t vocab, float scale,
                           int32_t dtype, int64_t stream);
/* out (dt_out) [T, width] (and out_f32, NULL or f32 [T, width]) = norm of the rows of x f32 [T, ldx] times w; kind 0: RMS, 1: layer
 * norm (mean taken off, variance = mean of the squared deviations) */
int mi355_hyb_pre_norm_ex(void* out, int32_t out_dtype, float* out_f32, const float* x, int32_t ldx, const float* w, int32_t num_tokens,
                          int32_t width, int32_t kind, float eps, int64_t stream);
/* mi355_hyb_gather_norm with the kind of norm as an argument */
int mi355_hyb_gather_norm_ex(void* out, int32_t out_dtype, const float* x, const int32_t* rows, const float* w, int32_t n_rows,
                             int32_t width, int32_t kind, float eps, int64_t stream);
/* x f32 [T, width] += a + b (b NULL: += a) */
int mi355_hyb_add2(float* x, const float* a, const float* b, int64_t n, int64_t stream);
/* x[t] += y[t] + sum_j weights[t, j] y_rows[pos[t top + j]]  (y NULL = none): the experts' weighted sum without a norm */
int mi355_hyb_moe_combine_add(float* x, const float* y, const float* y_rows, const int32_t* pos, const float* weights, int32_t num_tokens,
                              int32_t width, int32_t top, int64_t stream);
/* out (dt_out) [T, ff] = relu(u)^2 */
int mi355_hyb_relu2(void* out, int32_t out_dtype, const float* u, int64_t n, int64_t stream);
/* x <- cap tanh(x / cap) */
int mi355_hyb_tanh_cap(float* x, float cap, int64_t n, int64_t stream);
/* out (dt_out) [T, n] = in f32 [T, n] times sigmoid(gate_in[t, c]) element by element, gate_in f32 rows of ldg */
int mi355_hyb_elem_gate(void* out, int32_t out_dtype, const float* in, const float* gate_in, int32_t ldg, int32_t num_tokens, int32_t n,
                        int64_t stream);
/* out (dt_out) [T, dim] = gelu_tanh(g[t, k]) * table (dt) [vocab, ldt] row ids[t], column col + k */
int mi355_hyb_side_act(void* out, int32_t out_dtype, const float* g, const void* table, int32_t ldt, int32_t col, const uint32_t* ids,
                       int32_t num_tokens, int32_t dim, int32_t vocab, int32_t dtype, int64_t stream);
/* xs f32 [terms, n]: xs[terms - 1] <- x (the newest result), then x <- sum_j w[j] xs[j] */
int mi355_hyb_depth_average(float* x, float* xs, const float* w, int32_t terms, int64_t n, int64_t stream);
/* the end of a layer and the start of the next in one launch: x += y / rms(y) * side_w (y NULL: nothing added); then, with depth_w,
 * mi355_hyb_depth_average over xs; then, with norm_w, out (dt_out) [T, width] (and out_f32, NULL or f32) = the norm of kind `kind` of
 * the new x times norm_w (what mi355_hyb_pre_norm_ex would give) */
int mi355_hyb_layer_tail(float* x, const float* y, const float* side_w, float* xs, const float* depth_w, int32_t terms, void* out, int32_t out_dtype,
                         float* out_f32, const float* norm_w, int32_t num_tokens, int32_t width, int32_t kind, float eps, int64_t stream);
/* out (dt_out) [T, n] = (y * silu(gate_in[t, c])) / rms over each of `groups` equal parts * w[c]: the gate in front of the norm */
int mi355_hyb_gate_group_norm(void* out, int32_t out_dtype, const float* y, const float* gate_in, int32_t ldg, const float* w,
                              int32_t num_tokens, int32_t n, int32_t groups, float eps, int64_t stream);
/* state-space scan over the new tokens of every sequence, state f32 [slots] x [heads, n_state, vdim] (stride in floats).
 * xbc f32 [T, ldx]: x (heads x vdim) at 0, B (groups x n_state) behind it, C behind that, all behind the convolution and silu;
 * dt_in f32 rows of ldd: the raw step per head; dt = softplus(dt_in + dt_bias[h]), decay = exp(-exp(a_log[h]) dt);
 * S <- decay S + dt B x^T;  y f32 [T, heads, vdim] = S^T C + skip[h] x.  Head h reads group h / (heads / groups).  n_state <= 512. */
int mi355_hyb_ssd_scan(float* y, float* state, int64_t state_stride, const float* xbc, int32_t ldx, const float* dt_in, int32_t ldd,
                       const float* a_log, const float* dt_bias, const float* skip, const uint32_t* context_lens,
                       const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads,
                       int32_t groups, int32_t n_state, int32_t vdim, int64_t stream);
/* mi355_hyb_conv with a bias per channel (NULL = none) in front of the activation */
int mi355_hyb_conv_bias(float* out, const float* proj, int32_t ldp, int32_t off, const float* w, const float* bias, const float* conv_state,
                        int64_t state_stride, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                        const int32_t* token_seq, int32_t num_seqs, int32_t num_tokens, int32_t channels, int32_t taps, int32_t act,
                        int64_t stream);
/* mi355_hyb_masked_attention with a distance bias: dist f32 [2, heads] (NULL = none), score <- score - r1[h] ln(1 + r2[h] (i - j)) */
int mi355_hyb_biased_attention(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages,
                               const void* v_pages, const uint32_t* block_tables, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* token_seq, const float* sink, const float* dist,
                               int32_t num_seqs, int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                               int32_t block_size, int32_t max_blocks, int32_t window, int32_t keep_first, float scale, float out_scale,
                               int32_t k_ld, int32_t v_ld, float softcap, int32_t cross_values, int32_t dtype, int64_t stream);
/* mi355_hyb_latent_prepare with the query rows and the down-projection in buffers of their own: q_src f32 [T, ldq] holds per head
 * [dim | rot_dim] at q_off; c_src f32 [T, ldc] holds [kv_rank | rot_dim] at c_off.  pages NULL: nothing is cached (a layer that reads
 * another layer's pages) and c_src is not read */
int mi355_hyb_latent_prepare_ex(void* q_out, void* pages, const float* q_src, int32_t ldq, int32_t q_off, const float* c_src, int32_t ldc,
                                int32_t c_off, const float* q_abs, const float* c_norm_w, const float* cos_t, const float* sin_t,
                                const int64_t* positions, const int64_t* slot_mapping, int32_t num_tokens, int32_t heads, int32_t dim,
                                int32_t rot_dim, int32_t kv_rank, int32_t rot_dims, int32_t interleaved, float eps, int32_t dtype,
                                int64_t stream);
/* mi355_hyb_moe_route with the remaining switches: sigmoid_scores (s = sigmoid(z) instead of softmax), groups / keep_groups (> 0: only
 * experts of the keep_groups groups with the largest sum of their two best choice scores can be chosen), normalise (weights divided
 * by their sum + 1e-20 before the scale) */
int mi355_hyb_moe_route_ex(int32_t* expert_ids, float* weights, float* shared_gate, void* xn, int32_t out_dtype, const float* x,
                           const float* norm_w, const float* router, const float* correction, const float* gate_row, int32_t num_tokens,
                           int32_t width, int32_t experts, int32_t top, float scale, float eps, int32_t append_shared,
                           int32_t sigmoid_scores, int32_t groups, int32_t keep_groups, int32_t normalise, int64_t stream);
/* ---- mechanisms of the designs with several residual streams */
/* mi355_hyb_linear with an activation in the epilogue: columns < act_cols pass MI355_HYB_ACT_*; out (dt_out) [T, ldo] */
int mi355_hyb_linear_act(void* out, int32_t out_dtype, int32_t ldo, const void* a, int32_t a_dtype, int32_t lda, const void* w, const float* bias,
                         int32_t num_tokens, int32_t n, int32_t k, int32_t act, int32_t act_cols, int32_t dtype, int64_t stream);
/* mi355_hyb_linear_grouped with an activation on every column and the output type as an argument */
int mi355_hyb_linear_grouped_act(void* out, int32_t out_dtype, int32_t ldo, const void* a, int32_t a_dtype, int32_t lda, const int32_t* row_token,
                                 const void* w, int64_t w_bs, const int32_t* block_table, int32_t block_rows, int32_t n_blocks, int32_t n,
                                 int32_t k, int32_t act, int32_t dtype, int64_t stream);
/* mi355_hyb_biased_attention with the kind of mask (MI355_HYB_MASK_*; the window is the chunk's size for the chunked one) */
int mi355_hyb_attention(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages, const void* v_pages,
                        const uint32_t* block_tables, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* token_seq,
                        const float* sink, const float* dist, int32_t num_seqs, int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim,
                        int32_t vdim, int32_t block_size, int32_t max_blocks, int32_t mask_kind, int32_t window, int32_t keep_first,
                        float scale, float out_scale, int32_t k_ld, int32_t v_ld, float softcap, int32_t cross_values, int32_t dtype,
                        int64_t stream);
/* mi355_hyb_moe_route_ex with a bias on the logits (router_bias f32 [experts] or NULL) and one more kind of scores: score_kind 0 =
 * softmax, 1 = sigmoid, 2 = the experts are chosen by their logits (+ correction) and, with normalise, weighted by the softmax over the
 * chosen logits.  append_shared without a gate_row: the appended pair has weight 1 */
int mi355_hyb_moe_route_biased(int32_t* expert_ids, float* weights, float* shared_gate, void* xn, int32_t out_dtype, const float* x,
                               const float* norm_w, const float* router, const float* router_bias, const float* correction, const float* gate_row,
                               int32_t num_tokens, int32_t width, int32_t experts, int32_t top, float scale, float eps, int32_t append_shared,
                               int32_t score_kind, int32_t groups, int32_t keep_groups, int32_t normalise, int64_t stream);
/* rows i32 [T]: (previous token mul_prev + token mul_cur) mod buckets, or `buckets` at a sequence's first token; the last token of every
 * sequence's portion is left in last_token (one 32-bit word per state slot, stride in words), where the next portion finds it */
int mi355_hyb_bigram_rows(int32_t* rows, int32_t* last_token, int64_t state_stride, const uint32_t* tokens, const uint32_t* context_lens,
                          const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t buckets,
                          int64_t mul_prev, int64_t mul_cur, int64_t stream);
/* x f32 [T, copies, width]: every copy = table (dt) row ids[t] times scale + bigram (dt) row bigram_rows[t] (bigram NULL: nothing added) */
int mi355_hyb_embed_streams(float* x, const void* table, const void* bigram, const int32_t* bigram_rows, const uint32_t* ids, int32_t num_tokens,
                            int32_t copies, int32_t width, int32_t vocab, float scale, int32_t dtype, int64_t stream);
/* the end of one sublayer and the start of the next in one launch, X f32 [T, streams, width]:
 *   y = y_dense + sum_j moe_w[t, j] moe_rows[moe_pos[t top + j]]        (y_dense f32 [T, width] or NULL, moe_rows or NULL)
 *   X_j <- sum_i mix[i, j] X_i + out_w[j] y                             (mix NULL: X stays, nothing was computed yet)
 *   sum f32 [T, width] = sum_j X_j                                      (NULL = not written)
 *   out (dt_out) [T, width] (and out_f32, NULL or f32) = RMSnorm(sum_i in_w[i] X_i) norm_w    (norm_w NULL: neither this nor X is written)
 * streams <= 16, width <= 12288 */
int mi355_hyb_stream_step(float* X, const float* y_dense, const float* moe_rows, const int32_t* moe_pos, const float* moe_w, int32_t top,
                          const float* mix, const float* out_w, float* sum, const float* in_w, const float* norm_w, void* out,
                          int32_t out_dtype, float* out_f32, int32_t num_tokens, int32_t streams, int32_t width, float eps, int64_t stream);
/* out (dt_out) [T, n] = y / rms over each of `groups` equal parts * w[c] * sigmoid(gate_in[t, c]): the gate behind the norm */
int mi355_hyb_norm_sigmoid_gate(void* out, int32_t out_dtype, const float* y, const float* gate_in, int32_t ldg, const float* w,
                                int32_t num_tokens, int32_t n, int32_t groups, float eps, int64_t stream);
/* linear attention with a constant decay per head over the new tokens of every sequence, state f32 [slots] x [heads, dim, vdim] (stride in
 * floats): S <- decay[h] S + k v^T, o f32 [T, heads, vdim] = S^T q.  qkv f32 [T, ldq] holds q, k (heads x dim) and v (heads x vdim) at their
 * offsets.  scratch != NULL: portions are cut into pieces of 64 tokens that are worked on side by side on the f32 matrix cores (needs
 * dim and vdim that are multiples of 16, dim <= 512, and the floats below); NULL: one scan over the tokens.  dim <= 512 */
int mi355_hyb_decay_attention(float* o, float* state, int64_t state_stride, const float* qkv, int32_t ldq, int32_t q_off, int32_t k_off,
                              int32_t v_off, const float* decay, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                              const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads, int32_t dim, int32_t vdim,
                              float* scratch, int64_t stream);
/* floats of `scratch` that suit a step of this size; 0: the scan suits it (few tokens per sequence, or sizes that only the scan serves) */
int64_t mi355_hyb_decay_attention_scratch(int32_t num_tokens, int32_t num_seqs, int32_t heads, int32_t dim, int32_t vdim);
/* ---- mechanisms of the designs with a norm per sublayer of the same residual, and time mixing */
/* a product whose column segments read different left operands: segment i (seg_rows[i] rows of w, multiples of 128, together n; HOST array, at
 * most 8) reads a + (first + i) a_stride elements; else as mi355_hyb_linear */
int mi355_hyb_linear_segments(float* out, int32_t ldo, const void* a, int32_t a_dtype, int32_t lda, int64_t a_stride, int32_t first, const void* w,
                              const float* bias, const int32_t* seg_rows, int32_t n_seg, int32_t num_tokens, int32_t n, int32_t k, int32_t dtype,
                              int64_t stream);
/* gate and up in one product with the activation (MI355_HYB_ACT_SILU or _GELU) behind it: w [2 ff, k] holds 16 gate rows, their 16 up rows, the
 * next 16 gate rows, ... (mi355_hyb_interleave_gate_up makes that order of [ff gate rows | ff up rows]; ff a multiple of 16); out (dt_out)
 * [T, ldo] = act(gate) up; a and w are both (dt) */
int mi355_hyb_linear_glu(void* out, int32_t out_dtype, int32_t ldo, const void* a, int32_t lda, const void* w, int32_t num_tokens, int32_t ff,
                         int32_t k, int32_t act, int32_t dtype, int64_t stream);
/* the same per block of a table (mi355_hyb_linear_grouped) */
int mi355_hyb_linear_grouped_glu(void* out, int32_t out_dtype, int32_t ldo, const void* a, int32_t lda, const int32_t* row_token, const void* w,
                                 int64_t w_bs, const int32_t* block_table, int32_t block_rows, int32_t n_blocks, int32_t ff, int32_t k, int32_t act,
                                 int32_t dtype, int64_t stream);
int mi355_hyb_interleave_gate_up(void* out, const void* in, int32_t matrices, int32_t ff, int32_t k, int32_t dtype, int64_t stream);
/* the end of one layer and the start of the next in one launch:
 *   x' = x + (y1 + (y2 or sum_j moe_w[t, j] moe_rows[moe_pos[t top + j]]))     (each part NULL = none) -> x_out (NULL: not written)
 *   h = RMSnorm(x') norm1 -> out1 (dt_out) [T, width];   RMSnorm(x') norm2 -> out2 (dt_out) (and out2_f32, NULL or f32)   (norm2 NULL: neither)
 *   mixture m < mixes: h + (h' - h) mu[m] -> out1 + (m + 1) seg_stride elements, h' = the h of the token before: of the same portion, or
 *   for its first token h_state (f32 rows per slot, stride in floats; zeros at position 0); h_last f32 [num_seqs, width] <- the h of every
 *   portion's last token (the caller moves it into h_state once nothing reads the old one: mi355_hyb_bonus_recurrence does)
 * norm1 NULL: only the sum.  x_out may be x only without mixtures.  width <= 16384 */
int mi355_hyb_pair_step(const float* x, const float* y1, const float* y2, const float* moe_rows, const int32_t* moe_pos, const float* moe_w,
                        int32_t top, float* x_out, const float* norm1, const float* norm2, void* out1, int64_t seg_stride, void* out2,
                        int32_t out_dtype, float* out2_f32, const float* mu, int32_t mixes, const float* h_state, int64_t state_stride,
                        float* h_last, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                        const int32_t* token_seq, int32_t num_tokens, int32_t width, float eps, int64_t stream);
/* log_w f32 [T, ldw] = -exp(sum_r w2t[r, c] tanh(z[t, r]) + w0[c]), w2t f32 [rank, channels] */
int mi355_hyb_lowrank_decay(float* log_w, int32_t ldw, const float* z, int32_t ldz, const float* w2t, const float* w0, int32_t num_tokens,
                            int32_t rank, int32_t channels, int64_t stream);
/* recurrence with a decay per key channel and a bonus for the current token over the new tokens of every sequence, state f32 [slots] x
 * [heads, dim, vdim] (stride in floats): o f32 [T, heads, vdim] = (S + diag(bonus) k v^T)^T r, then S <- diag(exp(log_w)) S + k v^T.
 * rkv f32 [T, ldq] holds r, k (heads x dim) and v (heads x vdim) at their offsets; log_w f32 [T, ldw] (heads x dim), bonus f32 [heads, dim].
 * row != NULL: row f32 [num_seqs, row_n] moves into row_state (f32 per slot, the same stride).  dim <= 512.  scratch != NULL (16-byte
 * aligned, the floats below; dim and vdim multiples of 16): portions are cut into pieces of 64 tokens that are worked on side by side on the
 * f32 matrix cores; NULL: one scan over the tokens */
int mi355_hyb_bonus_recurrence(float* o, float* state, int64_t state_stride, const float* rkv, int32_t ldq, int32_t r_off, int32_t k_off,
                               int32_t v_off, const float* log_w, int32_t ldw, const float* bonus, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads,
                               int32_t dim, int32_t vdim, const float* row, float* row_state, int32_t row_n, float* scratch, int64_t stream);
/* floats of `scratch` that suit a step of this size; 0: the scan suits it (few tokens per sequence, or sizes that only the scan serves) */
int64_t mi355_hyb_bonus_recurrence_scratch(int32_t num_tokens, int32_t num_seqs, int32_t heads, int32_t dim, int32_t vdim);
/* mi355_hyb_gated_norm with weights per head: head h's start at w + h w_ld (w_ld 0: the same for all heads) */
int mi355_hyb_gated_norm_heads(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const float* o, const float* w, int32_t w_ld,
                               const float* gate_in, int32_t ldg, int32_t gate, int32_t num_tokens, int32_t heads, int32_t vdim, float eps,
                               float out_scale, int64_t stream);
/* mi355_hyb_attn_prepare_ex / _whole with a query temperature (temp_coef 0 = none): the query at position p times 1 + temp_coef
 * ln(floor((p + 1) / temp_every) + 1); k_pages and v_pages NULL: the queries only (a layer that reads another layer's pages) */
int mi355_hyb_attn_prepare_temp(void* q_out, void* k_pages, void* v_pages, const float* proj, int32_t ldp, int32_t q_off, int32_t k_off,
                                int32_t v_off, const float* q_norm_w, const float* k_norm_w, const float* cos_t, const float* sin_t,
                                const int64_t* positions, const int64_t* slot_mapping, int32_t num_tokens, int32_t heads, int32_t kv_heads,
                                int32_t dim, int32_t vdim, int32_t rot_dims, int32_t interleaved, int32_t norm_mode, const float* q_head_scale,
                                float temp_coef, float temp_every, float eps, int32_t dtype, int64_t stream);
int mi355_hyb_attn_prepare_whole_temp(void* q_out, void* k_pages, void* v_pages, const float* src, int32_t ld, int32_t q_off, int32_t k_off,
                                      int32_t v_off, const float* q_norm_w, const float* k_norm_w, const int64_t* positions,
                                      const int64_t* slot_mapping, int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                      int32_t v_unit, float temp_coef, float temp_every, float eps, int32_t dtype, int64_t stream);
/* mi355_hyb_attention with a linear distance bias (dist_linear: score - r1[h] (i - j)) and an output gate: head h's output of token t times
 * sigmoid(gate[t ldg + h]) (gate NULL = none) */
int mi355_hyb_attention_ex(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const void* q, const void* k_pages, const void* v_pages,
                           const uint32_t* block_tables, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* token_seq,
                           const float* sink, const float* dist, int32_t dist_linear, const float* gate, int32_t ldg, int32_t num_seqs,
                           int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size, int32_t max_blocks,
                           int32_t mask_kind, int32_t window, int32_t keep_first, float scale, float out_scale, int32_t k_ld, int32_t v_ld,
                           float softcap, int32_t cross_values, int32_t dtype, int64_t stream);
/* 0: prompt-sized steps over bf16 pages take the generic kernel instead of the matrix-core ones; 2: the matrix-core kernel with one
 * wave per head also where the query heads of a key/value head could share a workgroup (A/B switch, process-wide; default 1) */
void mi355_hyb_set_attention_mfma(int32_t on);
/* short causal convolution over time per channel, then silu: out f32 [T, channels] from proj columns [off, off + channels);
 * the taps - 1 inputs before a portion come from conv_state f32 [slots, channels, taps - 1] (zeros at position 0);
 * mi355_hyb_conv_state_update then moves the state behind the portion */
int mi355_hyb_conv_silu(float* out, const float* proj, int32_t ldp, int32_t off, const float* w, const float* conv_state,
                        int64_t state_stride, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                        const int32_t* state_slots, const int32_t* token_seq, int32_t num_seqs, int32_t num_tokens, int32_t channels,
                        int32_t taps, int64_t stream);
int mi355_hyb_conv_state_update(float* conv_state, int64_t state_stride, const float* proj, int32_t ldp, int32_t off,
                                const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                                int32_t num_seqs, int32_t channels, int32_t taps, int64_t stream);
/* gated delta rule over the new tokens of every sequence, state f32 [slots] x [heads, dim, vdim] (stride in floats).
 * qkv f32 [T, ldq]: q at 0 (kv_heads x dim, raw), k behind it, v behind that (heads x vdim); q and k are made unit vectors per head
 * (eps inside the root), q times dim^-1/2.  beta = sigmoid(proj[:, b_off + head]).  decay = exp(-exp(a_log[head]) * softplus(da +
 * dt_bias)) with da = decay_in[t, head] (channels = 0) or decay_in[t, head * dim + channel].  o f32 [T, heads, vdim]. */
int mi355_hyb_delta_rule(float* o, float* state, int64_t state_stride, const float* qkv, int32_t ldq, const float* proj,
                         int32_t ldp, int32_t b_off, const float* decay_in, int32_t ldd, int32_t decay_channels,
                         const float* a_log, const float* dt_bias, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                         const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim,
                         int32_t vdim, float unit_eps, float* scratch, int64_t stream);
/* floats of `scratch` (device): what the rule computes for all tokens at once before the scan over them */
int mi355_hyb_delta_rule_scratch_floats(int32_t num_tokens, int32_t heads, int32_t kv_heads, int32_t dim, int32_t decay_channels);
/* out (dt_out) [T, ldo] at out_off = o / rms(o over vdim) * w * gate(gate_in) * out_scale; gate: MI355_HYB_GATE_* (silu / sigmoid) */
int mi355_hyb_gated_norm(void* out, int32_t out_dtype, int32_t ldo, int32_t out_off, const float* o, const float* w,
                         const float* gate_in, int32_t ldg, int32_t gate, int32_t num_tokens, int32_t heads, int32_t vdim, float eps,
                         float out_scale, int64_t stream);
/* minGRU over the new tokens: z = sigmoid(proj[:, z_off + c]), u = proj[:, x_off + c], candidate = u + 1/2 (u >= 0) or sigmoid(u),
 * S = (1 - z) S + z candidate, out (dt_out) [T, width] = S silu(proj[:, g_off + c]); state f32 [slots] x [width] */
int mi355_hyb_mingru(void* out, int32_t out_dtype, float* state, int64_t state_stride, const float* proj, int32_t ldp, int32_t z_off,
                     int32_t x_off, int32_t g_off, const uint32_t* context_lens, const uint32_t* cu_seqlens_q,
                     const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t width, int64_t stream);
/* out (dt_out) [T, ff] = g sigmoid(alpha g) (u + 1), g = min(gu[:, j], limit), u = clamp(gu[:, ff + j], -limit, limit) */
int mi355_hyb_clamped_glu(void* out, int32_t out_dtype, const float* gu, int32_t num_tokens, int32_t ff, float limit, float alpha,
                          int64_t stream);

#ifdef __cplusplus
}
#endif
