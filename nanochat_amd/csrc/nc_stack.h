// Internal launch functions of the layer-stack library (include/nanochat_amd_stack.h).  Every function enqueues work on the given
// stream, never synchronises, never allocates, and returns 0 or a negative code after nc_set_error().
//
// Storage types: T is bf16_t (raw bfloat16) or float; `dtype` 0 / 1 selects it at run time.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "nc_common.h"
#include "nc_kernels.h"

// timing classes of NcProfScope / nc_profile_*
enum { NC_CLS_LATENT = 0, NC_CLS_LINEAR = 1, NC_CLS_RETENTION = 2, NC_CLS_ROWS = 3, NC_CLS_EXPERTS = 4, NC_CLS_WINDOW = 5, NC_CLS_SCAN = 6 };

// ---------------------------------------------------------------- element helpers
template <typename T> __device__ __forceinline__ float ld_f32(const T* p);
template <> __device__ __forceinline__ float ld_f32<bf16_t>(const bf16_t* p) { return bf16_to_f32(*p); }
template <> __device__ __forceinline__ float ld_f32<float>(const float* p) { return *p; }
__device__ __forceinline__ void st_f32(bf16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ void st_f32(float* p, float v) { *p = v; }
// four consecutive values
__device__ __forceinline__ v4f ld4_f32(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return v4f{bf16_lo(u.x), bf16_hi(u.x), bf16_lo(u.y), bf16_hi(u.y)};
}
__device__ __forceinline__ v4f ld4_f32(const float* p) { return *(const v4f*)p; }
__device__ __forceinline__ void st4_f32(bf16_t* p, v4f v) { *(uint2*)p = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])); }
__device__ __forceinline__ void st4_f32(float* p, v4f v) { *(v4f*)p = v; }

__device__ __forceinline__ float gelu_tanh_f32(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
__device__ __forceinline__ float sigmoid_f32(float z) { return __builtin_amdgcn_rcpf(1.0f + expf(-z)); }
// max(z, 0) + log(1 + e), e = exp(-|z|).  The exponential is one exp2 with the rounding of its argument put right to first order; the logarithm
// is 2 artanh(s), s = e / (2 + e) <= 1/3, by its series, so that a small e keeps all its digits.
__device__ __forceinline__ float softplus_f32(float z) {
    const float a = -fabsf(z), p = a * 1.44269504f, left = fmaf(a, 1.44269504f, -p) + a * 1.92596299e-8f;
    const float e2 = __builtin_amdgcn_exp2f(p), e = fmaf(e2, left * 0.693147181f, e2);
    const float s = e * __builtin_amdgcn_rcpf(2.f + e), q = s * s;
    float t = 1.f / 17.f;
#pragma unroll
    for (int k = 15; k >= 1; k -= 2) t = fmaf(t, q, 1.f / (float)k);
    return fmaf(2.f * s, t, fmaxf(z, 0.f));
}
__device__ __forceinline__ float silu_f32(float z) { return z * sigmoid_f32(z); }
// gate and up of one unit -> its activation, both clamped: the gate from above, up on both sides
__device__ __forceinline__ float clamped_glu_f32(float gate, float up, float limit) {
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g * sigmoid_f32(1.702f * g) * (u + 1.0f);
}

// ---------------------------------------------------------------- linears (nc_stack_gemm.hip)
// Where a run of output columns goes, and what happens to it on the way.
enum NcSegKind {
    NC_SEG_PLAIN = 0,      // T
    NC_SEG_GELU = 1,       // T, tanh-form gelu
    NC_SEG_GLU = 2,        // T, clamped GLU of interleaved columns (gate, up): half as many outputs
    NC_SEG_F32 = 3,        // float
    NC_SEG_RESIDUAL = 4,   // float, added to what is there
    NC_SEG_LOGITS = 5,     // float, p0 * v, then p1 * tanh(. / p1) if p1 > 0; bounds checked column by column
    NC_SEG_SILU = 6,       // T, silu
    NC_SEG_SWIGLU = 7,     // T, silu(gate) * up of interleaved columns (gate, up): half as many outputs
    NC_SEG_SOFTPLUS = 8,   // float, softplus(v + bias)
};
struct NcSeg {
    int end;               // exclusive last column (of the stacked weight) of this run
    int kind;
    void* out;             // output column 0 of the run
    int ld;                // elements between output rows
    float p0, p1;          // GLU: p0 = limit
    const float* bias;     // SOFTPLUS: per output column of the run
};
// The rows a linear works on: M rows of A; or, per batch, the same M with strides; or groups of rows, one group per weight (experts).
struct NcLinear {
    const void* a;
    int64_t lda;
    const void* w;         // [N, K], rows ldw elements apart
    int64_t ldw;
    int M, N, K;
    int nseg;
    NcSeg seg[4];
    int batch;                             // >= 1: how many (A, W, out) triples the strides (in elements) walk
    int64_t a_stride, w_stride, out_stride;
    // groups: tile t of `tiles` is {group, first row, rows, first tile of the group, tiles of the group}; the weight of group g starts w_stride * g elements on; row r of A is
    // a_rows[r] / a_div (or r itself without a_rows), row r of the output is r
    const int32_t* tiles;
    const int32_t* n_tiles;
    int max_tiles, tile_rows;
    const int32_t* a_rows;
    int a_div;
    // the few-rows kernel may leave fp32 partial sums [splits][M][N] for its consumer instead of finishing
    float* partials;
    int splits;
};
inline NcLinear nc_linear(const void* a, int64_t lda, const void* w, int M, int N, int K) {
    NcLinear l{};
    l.a = a, l.lda = lda, l.w = w, l.ldw = K, l.M = M, l.N = N, l.K = K, l.batch = 1, l.a_div = 1, l.splits = 1;
    return l;
}
inline void nc_linear_seg(NcLinear& l, int end, int kind, void* out, int ld, float p0 = 0.f, float p1 = 0.f, const float* bias = nullptr) {
    l.seg[l.nseg++] = NcSeg{end, kind, out, ld, p0, p1, bias};
}
#define NC_FEW_ROWS 64                     // up to here the few-rows kernel
#define NC_TILE_WORDS 5
#define NC_GROUP_TILE_FEW 16               // rows per group tile of the few-rows kernel (the tiled one takes 64 or 128)
int nc_launch_linear_few(int dtype, const NcLinear& l, hipStream_t s, int cls = NC_CLS_LINEAR);
int nc_launch_linear_tiled(int dtype, const NcLinear& l, hipStream_t s, int cls = NC_CLS_LINEAR, int shape = 0);     // shape 0: choose
// splits of the summed index over workgroups that fill the chip for a few-rows linear whose consumer adds partial sums
int nc_linear_few_splits(int M, int N, int K);

// ---------------------------------------------------------------- row kernels (nc_stack_rows.hip)
// What the rows that leave for the next linear are: layer norm or RMS norm of x times a weight, or x itself in the storage type.
enum NcRowNorm { NC_ROW_LAYER_NORM = 0, NC_ROW_RMS_NORM = 1, NC_ROW_COPY = 2 };
// x = embedding rows * scale (+ step); h = norm(x)
int nc_launch_stack_embed(int dtype, const int64_t* idx, const void* embed, float scale, const float* step, int vocab, float* x, float* x0,
                          int norm, const float* norm_w, float eps, void* h, int M, int width, int width_p, hipStream_t s);
// y = partial sums + weighted expert rows; x += y, or (post_norm_w) x += rms_norm(y) * post_norm_w; tap = x; x += x0 + step; h = norm(x).
// Rows may be a selection (`rows`: which row of x is normalised into row i of h); then x itself is not stored.
struct NcRowAdd {
    float* x;
    const float* partials;         // [splits][M][width_p] or null
    int splits;
    const void* expert_out;        // T [slots][width_p] or null
    const int32_t* slot_of;        // [M][top]
    const float* slot_w;           // [M][top]
    int top;
    const float* post_norm_w;      // or null
    float* tap;                    // [M][width_p] or null
    const float* x0;               // or null
    const float* step;             // or null
    int norm;                      // NcRowNorm of h
    const float* norm_w;
    void* h;
    const int32_t* rows;           // selection or null
    int32_t* bump;                 // cache positions to advance (one per batch row, by the row's last token) or null
    int bump_by, tokens_per_row;
};
int nc_launch_stack_row_add(int dtype, const NcRowAdd& a, float eps, int M, int n_rows, int width, int width_p, hipStream_t s);

// Expert choice: softmax over `experts` logits per row, the largest `top`, weights = their scores over their sum; then the (row, choice)
// pairs are put in expert order: perm[slot] = row * top + choice, slot_of its inverse, and tiles of `tile_rows` rows per expert.
struct NcRoute {
    const float* logits;           // [M][ld]
    int ld, experts, top;
    float* slot_w;                 // [M][top]
    int32_t* chosen;               // [M][top]
    int32_t* slot_of;              // [M][top]
    int32_t* perm;                 // [M * top]
    int32_t* tiles;                // [max_tiles][NC_TILE_WORDS], see NcLinear
    int32_t* n_tiles;
    int tile_rows, max_tiles;
};
int nc_launch_stack_route(const NcRoute& r, int M, hipStream_t s);
int nc_launch_stack_cache_copy(const void* src, void* dst, int src_rows, int dst_rows, int64_t src_stride, int64_t dst_stride, int64_t bytes,
                               hipStream_t s);

// ---------------------------------------------------------------- latent attention (nc_latent_attention.hip)
struct NcLatentGeom {
    int heads, dim_p, rot_p, rot_dims, rank, rank_p, vdim_p;
    float scale;
    int B, T, Tmax, pos_max;       // rows of the cache, new tokens per row, cache length, largest position before this call
};
// Normed latent and rotated shared key of the new tokens into the cache; the rotated part of the queries in place, or (q_lat != null)
// into q_lat[(m * heads + head)][rank_p ..].
int nc_launch_latent_append(int dtype, const NcLatentGeom& g, void* proj, int ldp, const float* norm_w, float eps, const float* rope,
                            int rope_len, const int32_t* seqlens, void* cache, void* q_lat, hipStream_t s);
// Attention in latent space: queries q_lat [M * heads][rank_p + rot_p], one cached vector per key that is key and value of all heads;
// out_lat T [M * heads][rank_p].
size_t nc_latent_partial_bytes(int dtype, const NcLatentGeom& g);
int nc_launch_latent_attention(int dtype, const NcLatentGeom& g, const void* q_lat, const void* cache, const int32_t* seqlens, void* out_lat,
                               void* partials, size_t partial_bytes, hipStream_t s);
// Attention over keys and values expanded per head: kv T [B][keys][heads * (dim_p + vdim_p)], rotated key parts from the cache.
bool nc_latent_expanded_ok(int dtype, const NcLatentGeom& g);
int nc_launch_latent_expanded(const NcLatentGeom& g, const bf16_t* q, int ldq, const bf16_t* kv, int keys, const bf16_t* cache,
                              const int32_t* seqlens, bf16_t* out, int ldo, hipStream_t s);

// ---------------------------------------------------------------- retention (nc_retention.hip)
struct NcRetentionGeom {
    int heads, dim, dim_p, vdim, vdim_p, rot_dims;
    float k_scale;
    int B, T;
    float* raw;                    // fp32 [B*T][heads * vdim_p]: the heads' outputs as they are go here instead of into `out`; or null
};
// proj: q | k | v | gate; out: normed per head, times silu(gate)
size_t nc_retention_workspace_bytes(int dtype, const NcRetentionGeom& g);
int nc_launch_retention(int dtype, const NcRetentionGeom& g, const void* proj, int ldp, const float* decay, const float* rope, int rope_len,
                        const int32_t* seqlens, const float* state_in, float* state_out, float eps, void* out, int ldo, void* workspace,
                        hipStream_t s);
// out = rms_norm(raw row, over `count` values of its `cols`) * w * sigmoid(gate) * scale
int nc_launch_joint_gate(int dtype, const float* raw, int cols, int count, const void* gate, int ldg, const float* w, float eps, float scale, void* out,
                         int ldo, int M, hipStream_t s);

// ---------------------------------------------------------------- window attention (nc_window_attention.hip)
struct NcWindowGeom {
    int heads, kv_heads, dim, dim_p, vdim_p, rot_dims;
    int window, keep_first;        // query i sees key j <= i if i - j < window or j < keep_first
    float scale, out_scale;
    int B, T, Tmax, pos_max;
};
// New tokens: bias, norm over the whole projection, rotation; queries in place, keys and values into the cache.
int nc_launch_window_append(int dtype, const NcWindowGeom& g, void* proj, int ldp, const float* bias, const float* q_norm_w, const float* k_norm_w, float eps,
                            const float* rope, int rope_len, const int32_t* seqlens, void* cache, hipStream_t s);
size_t nc_window_partial_bytes(int dtype, const NcWindowGeom& g);
int nc_launch_window_attention(int dtype, const NcWindowGeom& g, const void* q, int ldq, const void* cache, const float* sink, const int32_t* seqlens, void* out,
                               int ldo, void* partials, size_t partial_bytes, hipStream_t s);

// ---------------------------------------------------------------- selective scan (nc_selective_scan.hip)
struct NcScanGeom {
    int inner, inner_p, state, state_p, taps, dt_rank_p;
    float out_scale;
    int B, T;
};
__host__ __device__ inline int nc_scan_bc_cols(int state_p) { return (state_p + 15) / 16 * 16; }      // columns of B (and of C) in the projected rows
// u = silu(causal convolution of x); the convolution's part of the state moves on
int nc_launch_scan_conv(int dtype, const NcScanGeom& g, const void* x, int ldx, const float* w, const float* b, const int32_t* seqlens, const float* state_in,
                        float* state_out, void* u, hipStream_t s);
// The product that gives a token its step (before W_dt), B and C has few columns and a long sum: it is left in `splits` shares,
// parts fp32 [splits][M][dt_rank_p + 2 * nc_scan_bc_cols].  nc_launch_scan_join adds them up into dtr T [M][dt_rank_p] and bc fp32
// [M][2 * nc_scan_bc_cols].
int nc_launch_scan_join(int dtype, const NcScanGeom& g, const float* parts, int splits, void* dtr, float* bc, hipStream_t s);
// One token per row (T = 1): everything from those shares on in one launch.
struct NcScanStep {
    const float* parts;
    int splits;
    const void* w_dt_t;            // T [dt_rank_p][inner_p]
    const float *dt_b, *a_log2, *skip;
    const void *u, *z;
    int ldz;
    const int32_t* seqlens;
    const float* state_in;
    float* state_out;
    void* out;
    int ldo;
};
int nc_launch_scan_step(int dtype, const NcScanGeom& g, const NcScanStep& p, hipStream_t s);
// the recurrence and what follows it: out = (sum_n S C + skip u) * silu(z) * scale.  dt fp32 [M][inner_p], bc as above
size_t nc_scan_workspace_bytes(const NcScanGeom& g);
int nc_launch_scan(int dtype, const NcScanGeom& g, const void* u, const float* dt, const float* bc, const float* a_log2, const float* skip,
                   const void* z, int ldz, const int32_t* seqlens, const float* state_in, float* state_out, void* out, int ldo, void* workspace,
                   hipStream_t s);
