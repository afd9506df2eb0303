/*
 * nanollama_stack.h -- C ABI of libnanollama_stack.so: decoder-only models described layer by layer (MI355X, gfx950).
 *
 * The library exports the entry points of nanollama_hip.h that a serving host calls on a model -- nl_upload_tensor, nl_finalize,
 * nl_destroy, nl_last_error, nl_reset, nl_forward, nl_forward_argmax, nl_host_logits, nl_decode_greedy, nl_sample_decode, nl_prefill,
 * nl_forward_batch, nl_get_config, nl_synchronize, nl_timer_start / _stop, nl_memory_usage, nl_debug_read, nl_build_info,
 * nl_device_count, nl_abi_version -- with the same contracts, on handles made by nl_create_stack; the quantised Llama family lives
 * in libnanollama_hip.so behind the same names, so a host loads the library of the model's family and calls it the same way.
 * What differs for models with a recurrent state: a stream's positions run forward -- a call either starts at position 0 (the
 * state is then zero whatever the stream held) or goes on where the stream's last call ended; anything else is NL_ERR_STATE.
 *
 * A layer is up to three residual branches' worth of description:
 *     x += mix_scale terms of { attention(norm1 x), linear_attention(norm1 x) }        (either may be absent), or
 *     x += latent_attention(norm1 x)
 *     x += down(act(gate(norm2 x)) * up(norm2 x))                                      (absent when ff == 0)
 * With post_norm every sublayer's result goes through a norm of its own before it is added: x += norm1_post(mixer(norm1 x)), ....
 * Norms are x / sqrt(mean(x^2) + eps) * (1 + w), or * w with plain_norm.  Tensor names for nl_upload_tensor (matrices [out, in]):
 *     embed                                    [vocab, dim]     token table; also the output matrix unless untied
 *     head                                     [vocab, dim]     output matrix (untied)
 *     final_norm                               [dim]
 *     layers.N.norm1 / norm2                   [dim]            and norm1_post / norm2_post with post_norm
 *     layers.N.attn.q / k / v / g / o          query, key, value, gate, output;  attn.q_norm / k_norm [head dim]
 *     layers.N.lin.q / k / v / g / o           likewise;  lin.a1 [rank, dim], lin.a2 [heads * dim, rank], lin.a2_bias, lin.norm [vdim]
 *     layers.N.latent.dq / q_norm / uq         [q_rank, dim], [q_rank], [heads * (dim + rot_dim), q_rank]
 *     layers.N.latent.dkv / kv_norm            [kv_rank + rot_dim, dim], [kv_rank]      (absent with kv_from)
 *     layers.N.latent.uk / uv / o              [heads * dim, kv_rank], [heads * vdim, kv_rank], [dim, heads * vdim]
 *     layers.N.latent.sink / g                 [heads], [heads, dim]
 *     layers.N.ff.gate / up / down             and ff.gate_bias / up_bias / down_bias with ff_bias
 */
#ifndef NANOLLAMA_STACK_H
#define NANOLLAMA_STACK_H

#include "nanollama_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

#define NL_GGML_BF16 30 /* ggml's id of bfloat16; nl_upload_tensor takes NL_GGML_F32 and this */

/* softmax attention, score(i, j) = scale q_i.k_j - slope_h (i - j); heads == 0: absent */
typedef struct {
    int32_t heads, kv_heads, dim, vdim; /* query heads, key / value heads, query-key size, value size per head */
    int32_t window;                     /* query i attends keys i - window < j <= i; 0: no lower bound */
    int32_t qk_norm;                    /* per-head RMS norm of queries and keys, weights attn.q_norm / attn.k_norm */
    int32_t distance_bias;              /* slope_h = 2^(-8 (h + 1) / heads), else 0 */
    int32_t gate;                       /* output *= sigmoid(g h) before the output matrix */
    float scale;
    float mix_scale;                    /* factor of this branch in the layer's sum */
} nl_attn_desc;

/* gated linear attention, a decay per key channel sigmoid(a2 (a1 h) + bias)^(1 / tau); heads == 0: none */
typedef struct {
    int32_t heads, dim, vdim, rank;
    float tau;
    float mix_scale;
} nl_linattn_desc;

/* latent attention: c_q = norm(dq h), [qu_h, qr_h] = uq c_q, [c, r] = dkv h with c normed, qr_h and r rotated by position;
 * score_h = scale (qu_h . uk_h c + qr_h . r) over all earlier positions, values uv_h c; c and r are what is cached; heads == 0: none */
typedef struct {
    int32_t heads, dim, rot_dim, vdim;  /* per head: unrotated and rotated query-key size, value size */
    int32_t q_rank, kv_rank;
    int32_t kv_from;                    /* the earlier layer whose c and r (in its cache) this layer attends, -1: its own */
    int32_t rot_dims;                   /* rotated dimensions of rot_dim (even), the rest pass */
    int32_t rot_adjacent;               /* pairs are (2i, 2i + 1), else (i, i + rot_dims / 2) */
    int32_t sink;                       /* a learned score per head in the softmax's denominator */
    int32_t gate;                       /* head h's output *= sigmoid(g h)_h */
    float scale;
    double rope_base;
    double yarn_factor, yarn_original, yarn_fast, yarn_slow;   /* YaRN interpolation; yarn_factor 0: none */
} nl_latent_desc;

enum { NL_ACT_GELU_TANH = 0, NL_ACT_SILU = 1 };

typedef struct {
    nl_attn_desc attn;
    nl_linattn_desc lin;
    nl_latent_desc latent; /* not beside attn or lin */
    int32_t ff;            /* width of the gated feed-forward, 0: none */
    int32_t ff_act;        /* NL_ACT_* */
    int32_t ff_bias;       /* gate, up and down have biases */
} nl_layer_desc;

enum { NL_DTYPE_BF16 = 0, NL_DTYPE_F32 = 1 };

typedef struct {
    int32_t vocab, dim, n_layers;
    int32_t loop_start, loop_stop, loop_times; /* layers [start, stop) are a block that is executed `times` times; every execution of a
                                                  layer has a key / value ring and a state of its own, and from the second pass on the
                                                  block's input is x + (embedded tokens).  loop_times <= 1: every layer once */
    int32_t seq_len;        /* positions per stream (> 0) */
    int32_t max_streams;    /* 0 -> 1 */
    int32_t max_step_tokens;/* tokens of one launch sequence; longer prompts are cut (0 -> 2048) */
    int32_t device;
    int32_t dtype;          /* NL_DTYPE_BF16: products and activations in bfloat16, 32-bit accumulation, everything else 32-bit;
                               NL_DTYPE_F32: 32-bit throughout */
    int32_t flags;          /* NL_FLAG_NO_GRAPH */
    int32_t plain_norm;     /* norm gains are w instead of 1 + w */
    int32_t post_norm;      /* a norm behind every sublayer (not with a loop) */
    int32_t untied;         /* the output matrix is `head` */
    float eps, embed_scale;
} nl_stack_config;

NL_API int nl_create_stack(const nl_stack_config *cfg, const nl_layer_desc *layers, nl_handle *out);

/* One ragged step: entry i brings n_tokens[i] tokens of stream streams[i] (distinct) from position pos0[i] on; `tokens` holds them one
 * entry behind the other.  want[0 .. n_want) are indices into `tokens` (ascending) whose logits are stored to logits_out
 * [n_want][vocab].  next_ids (may be NULL) [n_entries]: argmax behind each entry's last token.  A step of one token per entry takes the
 * decode launches, anything else the prompt launches; of a model with latent attention, one-token entries take the decode launches and
 * the others the prompt launches.  The result of a token does not depend on which. */
NL_API int nl_step(nl_handle h, int n_entries, const int *streams, const int *n_tokens, const int *pos0, const int *tokens,
                   int n_want, const int *want, float *logits_out, int *next_ids);
/* Keep a copy of the residual stream behind every layer run of later calls (on != 0): nl_debug_read(h, "layers", 0, ...) returns
 * [layer runs][tokens of the last launch sequence][dim].  Graph replay is off while it is on. */
NL_API int nl_trace_layers(nl_handle h, int on);
#ifdef __cplusplus
}
#endif
#endif /* NANOLLAMA_STACK_H */
