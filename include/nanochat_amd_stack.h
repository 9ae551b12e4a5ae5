/* nanochat_amd layer stack -- C ABI of the decoder whose layers are listed in a configuration: any order of mixers (latent attention,
 * retention, window attention, selective scan, or two of them side by side) and feed-forwards (dense, mixture of experts), sublayers in
 * parallel behind one norm or one after the other with a norm on each output, a run of layers that may be repeated with the same weights,
 * in bfloat16 or in 32-bit throughout.  libnanochat_amd_stack.so; the conventions of nanochat_amd.h hold: device pointers unless a
 * parameter says "host", work enqueued on `stream`, nothing allocates or synchronises, 0 on success, negative on error with
 * nc_last_error().
 *
 * "T" below is the storage type of weights and activations: bfloat16 bits, or float.  32-bit in both: the residual stream, norms,
 * angles, attention scores and weights, router, recurrent state and all that enters it after the projections.
 *
 * Padding.  Every summed index is padded with zeros to a multiple of 64 (NC_STACK_PAD) and per-head sizes as the fields say, so that
 * no kernel needs a tail along it: weights carry zero rows / columns there, which makes the padded activations zero as well.
 */
#ifndef NANOCHAT_AMD_STACK_H
#define NANOCHAT_AMD_STACK_H
#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef void* nc_stream_t;

#define NC_STACK_PAD 64
enum { NC_MIXER_LATENT_ATTENTION = 0, NC_MIXER_RETENTION = 1, NC_MIXER_WINDOW_ATTENTION = 2, NC_MIXER_SELECTIVE_SCAN = 3 };
enum { NC_FF_NONE = 0, NC_FF_DENSE_GELU = 1, NC_FF_EXPERTS = 2, NC_FF_DENSE_SWIGLU = 3 };
/* How a layer's sublayers are put together:
 *   parallel   h = norm(x); x += mixer(h) + ff(h)
 *   post-norm  x += norm1(mixer(x)); x += norm2(ff(x)): the sublayers read x itself */
enum { NC_BLOCK_PARALLEL = 0, NC_BLOCK_POST_NORM = 1 };
enum { NC_NORM_LAYER = 0, NC_NORM_RMS = 1 };
/* What becomes of a retention head's outputs o: normed per head times silu(gate), or all heads normed together with a weight times
 * sigmoid(gate). */
enum { NC_GATE_HEAD_NORM_SILU = 0, NC_GATE_JOINT_NORM_SIGMOID = 1 };
#define NC_STACK_MAX_MIXERS 2

int nc_stack_abi_version(void);
const char* nc_last_error(void);

/* One mixer.  Its projections are `cols` rows of its layer's input matrix and `cols` columns of the projected rows:
 *   latent attention  q (heads x (dim_p + rot_p)) | latent (rank_p) | shared rotated key (rot_p)
 *   retention         q (heads x dim_p) | k (heads x dim_p) | v (heads x vdim_p) | gate (heads x vdim_p); silu_qkv: q, k, v pass silu
 *   window attention  q (heads x dim_p) | k (kv_heads x dim_p) | v (kv_heads x vdim_p)
 *   selective scan    x (inner_p) | z (inner_p)
 * and its result `out` columns of what the output matrix multiplies, times out_scale. */
typedef struct nc_stack_mixer {
    int kind, cols, out;
    int heads, dim, dim_p, vdim, vdim_p;
    int rot_dim, rot_p;             /* latent attention: size of the rotated part per head; rot_p a multiple of 32 */
    int rank, rank_p;               /* latent attention: size of the latent; rank_p a multiple of 64 */
    int rot_dims;                   /* how many leading dimensions of the rotated vector turn (a pair is (i, i + rot_dims/2)) */
    float score_scale;              /* attention: factor of the scores; retention: factor of k after its rotation */
    float out_scale;                /* window attention, joint-norm retention, selective scan; the others have 1 */
    int silu_qkv, gate;             /* retention */
    int kv_heads, window, keep_first; /* window attention: query i sees key j <= i if i - j < window or j < keep_first */
    int inner, inner_p, state, state_p, taps, dt_rank, dt_rank_p;    /* selective scan; state_p = 4, 8, 12 or 16 times a power of two (up to 16) */
    const float* kv_norm_w;         /* latent attention: fp32 [rank_p] */
    const void* w_uk_t;             /* latent attention: T [heads, rank_p, dim_p]: W_uk of each head, transposed */
    const void* w_ukv;              /* latent attention: T [heads * (dim_p + vdim_p), rank_p]: unrotated key and value rows of each head */
    const float* decay;             /* retention: fp32 [heads, 2]: decay, log2 of it (finite) */
    const float* rope;              /* fp32 [rope_len, rot_dims/2, 2]: cos, sin of position * frequency; NULL if rot_dims is 0 */
    const float* qkv_bias;          /* window attention: fp32 [cols] */
    const float* q_norm_w;          /* window attention: fp32 [heads * dim_p], the norm runs over all heads at once */
    const float* k_norm_w;          /* window attention: fp32 [kv_heads * dim_p] */
    const float* sink;              /* window attention: fp32 [heads]: exp(sink) counts in the softmax's denominator */
    const float* out_norm_w;        /* joint-norm retention: fp32 [heads * vdim_p] */
    const float* conv_w;            /* selective scan: fp32 [taps, inner_p], the last tap is the current token's */
    const float* conv_b;            /* selective scan: fp32 [inner_p] */
    const void* w_x;                /* selective scan: T [dt_rank_p + 2 * round16(state_p), inner_p]: step, B and C rows */
    const void* w_dt;               /* selective scan: T [inner_p, dt_rank_p] */
    const void* w_dt_t;             /* selective scan: T [dt_rank_p, inner_p]: the same transposed */
    const float* dt_b;              /* selective scan: fp32 [inner_p] */
    const float* a_log2;            /* selective scan: fp32 [state_p, inner_p]: A * log2(e), A < 0 */
    const float* skip;              /* selective scan: fp32 [inner_p] */
} nc_stack_mixer;

/* One layer.  Parallel block: both sublayers read h, so their first matrices are one weight (w_in) and their last ones, which add into x,
 * another (w_out):
 *   w_in  [n_in, width_p] rows:  the mixers' projections (mix_cols rows), then router logits (router_cols), then the feed-forward's
 *         first matrix (ff_cols rows: up, or gate and up interleaved row by row), each part padded to a multiple of 16 rows
 *   w_out [width_p, k_out] columns: the mixers' results (mix_out), then the feed-forward's ff_p
 * Post-norm block (dense feed-forward or none): w_in and w_out hold the mixers alone, w_ff_in [ff_cols, width_p] and w_ff_out
 * [width_p, ff_p] the feed-forward. */
typedef struct nc_stack_layer {
    int block, n_mixers, ff;
    int mix_cols, router_cols, ff_cols, n_in;
    int mix_out, ff_p, k_out;       /* ff_p: padded width of the dense layer, or of the shared expert (0: none) */
    float ff_limit;                 /* shared expert: clamp limit */
    int experts, top, expert_ff_p;
    float expert_limit;
    const float* norm_w;            /* fp32 [width_p]: of x in front of both sublayers, or of the mixers' result */
    const float* norm2_w;           /* fp32 [width_p]: of the feed-forward's result (post-norm block) */
    const void* w_in;
    const void* w_out;
    const void* w_ff_in;
    const void* w_ff_out;
    const void* w_e1;               /* T [experts, 2 * expert_ff_p, width_p]: gate and up interleaved row by row */
    const void* w_e2;               /* T [experts, width_p, expert_ff_p] */
    nc_stack_mixer mix[NC_STACK_MAX_MIXERS];
} nc_stack_layer;

/* The runs in order: layer index, cache slot of each mixer (0 .. slots of its kind of cache - 1) and what happens to x right before. */
typedef struct nc_stack_run {
    int layer, slot[NC_STACK_MAX_MIXERS];
    int add_embedding;              /* x += the embedding output */
    int step;                       /* >= 0: x += step vector `step` */
} nc_stack_run;

typedef struct nc_stack_model {
    int dtype;                      /* 0 bfloat16, 1 float */
    int width, width_p, vocab, rope_len, n_layers, n_runs, max_k_out, norm;      /* norm: of the whole model, NC_NORM_* */
    float eps, embed_scale, logit_scale, logit_softcap;      /* softcap 0: none */
    const void* embed;              /* T [vocab, width_p] */
    const void* head;               /* T [vocab, width_p] */
    const float* final_norm_w;      /* fp32 [width_p] */
    const float* steps;             /* fp32 [times, width_p] or NULL */
    const nc_stack_layer* layers;   /* HOST array */
    const nc_stack_run* runs;       /* HOST array */
} nc_stack_model;

/* Cache.  Token rows: T [slots][batch][max_seq_len][row width(slot)], one allocation per slot (host array of device pointers).  A row of
 * latent attention is rank_p latent values and rot_p of the rotated key; one of window attention, for every kv head, its dim_p key values
 * (normed and rotated) and vdim_p values.  States: fp32, two buffers per slot: a forward reads state_in and writes state_out (a caller
 * can take a step back by swapping them again); retention [batch][heads][dim_p][vdim_p], selective scan [batch][state_p + taps - 1][inner_p]
 * (the recurrent state, then the convolution's last inputs, oldest first).  A row at position 0 does not read its state.  cache_seqlens:
 * tokens cached before this call; the caller advances it. */
typedef struct nc_stack_cache {
    void* const* rows;              /* HOST array of device pointers, one per attention run */
    float* const* state_in;         /* HOST arrays of device pointers, one per run of a recurrent mixer */
    float* const* state_out;
    int32_t* cache_seqlens;
    int batch, max_seq_len;
    int pos_max;                    /* host copy of the largest cache_seqlens entry */
    int advance;                    /* != 0: the last row kernel adds it to every cache_seqlens entry */
} nc_stack_cache;

/* Workspace for one forward of T tokens per row, n_logits rows of logits, at most max_keys keys per row. */
size_t nc_stack_workspace_bytes(const nc_stack_model* model /*host*/, int B, int T, int n_logits, int max_keys);

/* idx int64 [B,T]; logit_rows int32 [n_logits]: flat indices (row * T + token) whose logits are wanted (device); logits_out fp32
 * [n_logits, vocab].  n_logits may be 0.  taps (or NULL): fp32 [n_runs, B*T, width_p], the residual stream after every run. */
int nc_stack_forward(const nc_stack_model* model /*host*/, const nc_stack_cache* cache /*host*/, const int64_t* idx, int B, int T,
                     const int32_t* logit_rows, int n_logits, float* logits_out, void* workspace, size_t workspace_bytes, float* taps,
                     nc_stream_t stream);

/* ---- the mechanisms one by one (what the forward launches; tests and other callers) ---------------------------------------------- */

/* out[M,N] (T, leading dimension ldc) = A[M,K] W[N,K]^T; kind 0 plain, 1 tanh-form gelu, 2 clamped GLU of interleaved (gate, up)
 * columns (N/2 outputs), 3 float output, 6 silu, 7 silu(gate) * up of interleaved columns (N/2 outputs).
 * kernel: 0 choose, 1 the few-rows kernel, 2 the tiled kernel, 3, 4 the tiled kernel with tiles of 64 x 128, 128 x 256.  K a multiple of 64, N of 16. */
int nc_stack_linear(int dtype, const void* a, int64_t lda, const void* w, void* out, int ldc, int M, int N, int K, int kind, float limit,
                    int kernel, nc_stream_t stream);

/* KVCache.prefill for one slot of either kind of cache: rows [0, n_bytes) of every batch row, src_rows 1 (broadcast) or dst_rows. */
int nc_stack_cache_copy(const void* src, void* dst, int src_rows, int dst_rows, int64_t src_row_bytes, int64_t dst_row_bytes,
                        int64_t n_bytes, nc_stream_t stream);

/* ---- measurement aid: see nanochat_amd.h.  Classes: 0 latent attention, 1 linears, 2 retention, 3 row kernels, 4 expert linears,
 * 5 window attention, 6 selective scan. -- */
int nc_profile_enable(int on);
int nc_profile_read(int cls, double* total_ms /*host*/, double* total_units /*host*/, int64_t* count /*host*/);
int nc_profile_read_gemm(int N, int K, double* total_ms /*host*/, double* total_units /*host*/, int64_t* count /*host*/);

#ifdef __cplusplus
}
#endif
#endif
