// Row kernels of the layer stack: embedding, residual add + norm, expert choice, cache copy.  The residual stream is fp32
// [M][width_p] (columns past `width` stay zero), norms are fp32, the normed rows leave in the storage type of the linears.
#include "nc_stack.h"

namespace {
constexpr int ROW_THREADS = 256;

// 1 / rms of one row held in registers, four columns per thread and step; columns past width hold 0
template <int STEPS>
__device__ __forceinline__ float inverse_rms(const v4f (&x)[STEPS], float eps, int width, float* red) {
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < STEPS; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) sq = fmaf(x[i][r], x[i][r], sq);
    return 1.0f / sqrtf(block_sum<ROW_THREADS / 64>(sq, red) / (float)width + eps);
}

// h[i] = norm(x)[i] of such a row: (x[i] - mean) / sqrt(var + eps) * w[i], or x[i] / rms(x) * w[i], or x[i]
template <typename T, int STEPS>
__device__ __forceinline__ void norm_row(int norm, const v4f (&x)[STEPS], const float* __restrict__ w, float eps, int width, int width_p, T* __restrict__ h,
                                         float* red) {
    float mean = 0.f, inv = 1.f;
    if (norm == NC_ROW_LAYER_NORM) {           // (uniform)
        float sum = 0.f, sq = 0.f;
#pragma unroll
        for (int i = 0; i < STEPS; i++) sum += (x[i][0] + x[i][1]) + (x[i][2] + x[i][3]);
        mean = block_sum<ROW_THREADS / 64>(sum, red) / (float)width;
#pragma unroll
        for (int i = 0; i < STEPS; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int c = 4 * ((int)threadIdx.x + i * ROW_THREADS) + r;
                const float d = x[i][r] - mean;
                sq += c < width ? d * d : 0.f;
            }
        inv = 1.0f / sqrtf(block_sum<ROW_THREADS / 64>(sq, red) / (float)width + eps);
    } else if (norm == NC_ROW_RMS_NORM) {
        inv = inverse_rms<STEPS>(x, eps, width, red);
    }
#pragma unroll
    for (int i = 0; i < STEPS; i++) {
        const int c = 4 * ((int)threadIdx.x + i * ROW_THREADS);
        if (c >= width_p) break;
        if (norm == NC_ROW_COPY) {
            st4_f32(h + c, x[i]);
            continue;
        }
        const v4f wv = *(const v4f*)(w + c);
        st4_f32(h + c, v4f{(x[i][0] - mean) * inv * wv[0], (x[i][1] - mean) * inv * wv[1], (x[i][2] - mean) * inv * wv[2], (x[i][3] - mean) * inv * wv[3]});
    }
}

template <typename T, int STEPS>
__global__ __launch_bounds__(ROW_THREADS) void stack_embed_kernel(const int64_t* __restrict__ idx, const T* __restrict__ embed, float scale,
                                                                  const float* __restrict__ step, int vocab, float* __restrict__ x,
                                                                  float* __restrict__ x0, int norm, const float* __restrict__ norm_w, float eps,
                                                                  T* __restrict__ h, int width, int width_p) {
    __shared__ float red[ROW_THREADS / 64];
    const int64_t m = blockIdx.x;
    int64_t id = idx[m];
    if (id < 0 || id >= vocab) id = 0;       // the caller checks the ids of a prompt; a bad one must not read outside the table
    v4f v[STEPS];
#pragma unroll
    for (int i = 0; i < STEPS; i++) {
        const int c = 4 * ((int)threadIdx.x + i * ROW_THREADS);
        v[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (c < width_p) {
            v[i] = ld4_f32(embed + id * width_p + c) * scale;
            if (x0) *(v4f*)(x0 + m * width_p + c) = v[i];
            if (step) v[i] += *(const v4f*)(step + c);
            *(v4f*)(x + m * width_p + c) = v[i];
        }
    }
    norm_row<T, STEPS>(norm, v, norm_w, eps, width, width_p, h + m * width_p, red);
}

// (every loop over splits and choices asks for its loads in batches, all of a batch before the first sum: a few rows' worth of these
// kernels lasts as long as its longest chain of dependent loads)
template <typename T, int STEPS>
__global__ __launch_bounds__(ROW_THREADS) void stack_row_add_kernel(NcRowAdd a, float eps, int M, int width, int width_p) {
    constexpr int BATCH = 8;
    __shared__ float red[ROW_THREADS / 64];
    const int64_t m = a.rows ? a.rows[blockIdx.x] : (int)blockIdx.x;
    v4f v[STEPS], y[STEPS];
#pragma unroll
    for (int i = 0; i < STEPS; i++) {
        const int c = 4 * ((int)threadIdx.x + i * ROW_THREADS);
        v[i] = c < width_p ? *(const v4f*)(a.x + m * width_p + c) : v4f{0.f, 0.f, 0.f, 0.f};
        y[i] = v4f{0.f, 0.f, 0.f, 0.f};
    }
    if (a.partials) {
#pragma unroll
        for (int i = 0; i < STEPS; i++) {
            const int at = 4 * ((int)threadIdx.x + i * ROW_THREADS), c = min(at, width_p - 4);
            v4f p[BATCH], sum = v4f{0.f, 0.f, 0.f, 0.f};
            for (int s0 = 0; s0 < a.splits; s0 += BATCH) {
#pragma unroll
                for (int s = 0; s < BATCH; s++) p[s] = *(const v4f*)(a.partials + ((int64_t)min(s0 + s, a.splits - 1) * M + m) * width_p + c);
#pragma unroll
                for (int s = 0; s < BATCH; s++)
                    if (s0 + s < a.splits) sum += p[s];
            }
            if (at < width_p) y[i] = sum;
        }
    }
    if (a.expert_out) {
        for (int k0 = 0; k0 < a.top; k0 += BATCH) {
            int64_t slot[BATCH];
            float w[BATCH];
#pragma unroll
            for (int k = 0; k < BATCH; k++) {
                const int64_t p = m * a.top + min(k0 + k, a.top - 1);
                slot[k] = a.slot_of[p];
                w[k] = a.slot_w[p];
            }
#pragma unroll
            for (int i = 0; i < STEPS; i++) {
                const int c = min(4 * ((int)threadIdx.x + i * ROW_THREADS), width_p - 4);
                v4f e[BATCH];
#pragma unroll
                for (int k = 0; k < BATCH; k++) e[k] = ld4_f32((const T*)a.expert_out + slot[k] * width_p + c);
#pragma unroll
                for (int k = 0; k < BATCH; k++)
                    if (k0 + k < a.top) y[i] += e[k] * w[k];
            }
        }
    }
    if (a.post_norm_w) {                       // (uniform; no expert rows here: y is zero past the padded width)
        const float inv = inverse_rms<STEPS>(y, eps, width, red);
#pragma unroll
        for (int i = 0; i < STEPS; i++) y[i] *= *(const v4f*)(a.post_norm_w + min(4 * ((int)threadIdx.x + i * ROW_THREADS), width_p - 4)) * inv;
    }
#pragma unroll
    for (int i = 0; i < STEPS; i++) v[i] += y[i];
#pragma unroll
    for (int i = 0; i < STEPS; i++) {
        const int c = 4 * ((int)threadIdx.x + i * ROW_THREADS);
        if (c >= width_p) {
            v[i] = v4f{0.f, 0.f, 0.f, 0.f};
            continue;
        }
        if (a.tap) *(v4f*)(a.tap + m * width_p + c) = v[i];
        if (a.x0) v[i] += *(const v4f*)(a.x0 + m * width_p + c);
        if (a.step) v[i] += *(const v4f*)(a.step + c);
        if (!a.rows) *(v4f*)(a.x + m * width_p + c) = v[i];
    }
    if (a.h) norm_row<T, STEPS>(a.norm, v, a.norm_w, eps, width, width_p, (T*)a.h + (int64_t)blockIdx.x * width_p, red);
    if (a.bump && threadIdx.x == 0 && (int)blockIdx.x % a.tokens_per_row == a.tokens_per_row - 1) a.bump[(int)blockIdx.x / a.tokens_per_row] += a.bump_by;
}

// ------------------------------------------------------------------------------------------------ expert choice
// One wave per row: lane l holds the scores of experts l, l + 64, ...; ties go to the lowest lane.
constexpr int ROUTE_MAX_EXPERTS = 1024;
// maximum over the wave: inside rows of 16 lanes without leaving the registers
__device__ __forceinline__ float row_wave_max(float v) {
    v = fmaxf(v, dpp_f32<0x128>(v));
    v = fmaxf(v, dpp_f32<0x124>(v));
    v = fmaxf(v, dpp_f32<0x122>(v));
    v = fmaxf(v, dpp_f32<0x121>(v));
    v = fmaxf(v, __shfl_xor(v, 16));
    return fmaxf(v, __shfl_xor(v, 32));
}
template <int PER>
__device__ __forceinline__ void choose_experts_of(const NcRoute& r, int m, int lane) {
    float s[PER];
    const float* z = r.logits + (int64_t)m * r.ld;
    float mx = -3.0e38f;
#pragma unroll
    for (int i = 0; i < PER; i++) {
        const int e = lane + 64 * i;
        s[i] = e < r.experts ? z[e] : -3.0e38f;
        mx = fmaxf(mx, s[i]);
    }
    mx = row_wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PER; i++) {
        const int e = lane + 64 * i;
        s[i] = e < r.experts ? expf(s[i] - mx) : -1.f;
        sum += e < r.experts ? s[i] : 0.f;
    }
    sum = wave_sum(sum);
    float chosen_sum = 0.f, mine = 0.f;       // lane k keeps the score of choice k (top <= 64)
    for (int k = 0; k < r.top; k++) {
        float best = -2.f;
        int at = 0;
#pragma unroll
        for (int i = 0; i < PER; i++)
            if (s[i] > best) best = s[i], at = lane + 64 * i;
        // (a row of NaN scores chooses experts 0, 1, ..: `best` keeps its start value)
        const float top = row_wave_max(best);
        at = __builtin_amdgcn_readlane(at, __ffsll((unsigned long long)__builtin_amdgcn_ballot_w64(best == top)) - 1);
        best = top;
        const float score = best / sum;
        chosen_sum += score;
        if (lane == k) mine = score;
        if (lane == 0) r.chosen[m * r.top + k] = at;
#pragma unroll
        for (int i = 0; i < PER; i++)
            if (at == lane + 64 * i) s[i] = -1.5f;
    }
    if (lane < r.top) r.slot_w[m * r.top + lane] = mine / (chosen_sum + 1e-20f);
}

__device__ __forceinline__ void choose_experts(const NcRoute& r, int m, int lane) {
    if (r.experts <= 64) choose_experts_of<1>(r, m, lane);
    else if (r.experts <= 256) choose_experts_of<4>(r, m, lane);
    else choose_experts_of<ROUTE_MAX_EXPERTS / 64>(r, m, lane);
}

__global__ __launch_bounds__(256) void route_choose_kernel(NcRoute r, int M) {
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (m < M) choose_experts(r, m, threadIdx.x & 63);
}

// The (row, choice) pairs in expert order: one workgroup counts, scans and deals out.  CHOOSE: it makes the choices first (few rows).
// (The order of the pairs inside an expert is whatever the atomics give: every pair is a row of its own, so no result depends on it.)
template <bool CHOOSE>
__global__ __launch_bounds__(1024) void route_sort_kernel(NcRoute r, int M) {
    __shared__ int count[ROUTE_MAX_EXPERTS], start[ROUTE_MAX_EXPERTS];
    const int pairs = M * r.top;
    for (int e = threadIdx.x; e < r.experts; e += 1024) count[e] = 0;
    if (CHOOSE)
        for (int m = threadIdx.x >> 6; m < M; m += 16) choose_experts(r, m, threadIdx.x & 63);
    __syncthreads();          // (also makes the choices of all waves, global stores of this workgroup, visible to it)
    for (int p = threadIdx.x; p < pairs; p += 1024) atomicAdd(&count[r.chosen[p]], 1);
    __syncthreads();
    // exclusive sums over the experts of rows and of tiles, by one wave, 64 experts at a time
    if (threadIdx.x < 64) {
        const int lane = threadIdx.x;
        int rows_before = 0, tiles_before = 0;
        for (int e0 = 0; e0 < r.experts; e0 += 64) {
            const int e = e0 + lane, c = e < r.experts ? count[e] : 0, t = (c + r.tile_rows - 1) / r.tile_rows;
            int cs = c, ts = t;
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const int c2 = __shfl_up(cs, o), t2 = __shfl_up(ts, o);
                if (lane >= o) cs += c2, ts += t2;
            }
            if (e < r.experts) {
                const int row0 = rows_before + cs - c, tile0 = tiles_before + ts - t;
                start[e] = row0;
                for (int i = 0; i < t; i++) {
                    int32_t* tile = r.tiles + NC_TILE_WORDS * (tile0 + i);
                    tile[0] = e, tile[1] = row0 + i * r.tile_rows, tile[2] = min(r.tile_rows, c - i * r.tile_rows), tile[3] = tile0, tile[4] = t;
                }
            }
            rows_before += __shfl(cs, 63), tiles_before += __shfl(ts, 63);
        }
        if (lane == 0) *r.n_tiles = tiles_before;
    }
    __syncthreads();
    for (int p = threadIdx.x; p < pairs; p += 1024) {
        const int slot = atomicAdd(&start[r.chosen[p]], 1);
        r.perm[slot] = p;
        r.slot_of[p] = slot;
    }
}

// ------------------------------------------------------------------------------------------------ joint norm and gate
// One workgroup per row; the row passes twice, the second time out of the cache.
template <typename T>
__global__ __launch_bounds__(256) void joint_gate_kernel(const float* __restrict__ raw, int cols, int count, const T* __restrict__ gate, int ldg,
                                                         const float* __restrict__ w, float eps, float scale, T* __restrict__ out, int ldo) {
    __shared__ float red[4];
    const int64_t m = blockIdx.x;
    const float* o = raw + m * cols;
    float sq = 0.f;
    for (int c = 4 * threadIdx.x; c < cols; c += 1024) {
        const v4f v = *(const v4f*)(o + c);
        sq += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    const float inv = scale / sqrtf(block_sum<4>(sq, red) / (float)count + eps);
    for (int c = 4 * threadIdx.x; c < cols; c += 1024) {
        const v4f v = *(const v4f*)(o + c), g = ld4_f32(gate + m * ldg + c), wv = *(const v4f*)(w + c);
        st4_f32(out + m * ldo + c, v4f{v[0] * inv * wv[0] * sigmoid_f32(g[0]), v[1] * inv * wv[1] * sigmoid_f32(g[1]), v[2] * inv * wv[2] * sigmoid_f32(g[2]),
                                       v[3] * inv * wv[3] * sigmoid_f32(g[3])});
    }
}

__global__ __launch_bounds__(256) void stack_cache_copy_kernel(const uint8_t* __restrict__ src, uint8_t* __restrict__ dst, int src_rows,
                                                               int64_t src_stride, int64_t dst_stride, int64_t pieces) {
    const int row = blockIdx.y;
    const uint4* s = (const uint4*)(src + (src_rows == 1 ? 0 : row) * src_stride);
    uint4* d = (uint4*)(dst + row * dst_stride);
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < pieces; i += (int64_t)gridDim.x * 256) d[i] = s[i];
}

// columns per thread: 4 per step of 1024 columns
#define STEPS_SWITCH(width_p, CALL)                      \
    do {                                                 \
        const int st__ = ((width_p) + 1023) / 1024;      \
        if (st__ <= 1) { CALL(1); }                      \
        else if (st__ <= 2) { CALL(2); }                 \
        else if (st__ <= 4) { CALL(4); }                 \
        else { CALL(8); }                                \
    } while (0)
}  // namespace

int nc_launch_stack_embed(int dtype, const int64_t* idx, const void* embed, float scale, const float* step, int vocab, float* x, float* x0,
                          int norm, const float* norm_w, float eps, void* h, int M, int width, int width_p, hipStream_t s) {
    NC_CHECK_ARG(width_p % 4 == 0 && width <= width_p && width_p <= 8192, "stack_embed: width %d", width_p);
    NcProfScope prof(NC_CLS_ROWS, (double)M * width_p * 8, s);
#define CALL(S)                                                                                                                                \
    if (dtype) hipLaunchKernelGGL((stack_embed_kernel<float, S>), dim3(M), dim3(ROW_THREADS), 0, s, idx, (const float*)embed, scale, step, vocab, \
                                  x, x0, norm, norm_w, eps, (float*)h, width, width_p);                                                              \
    else hipLaunchKernelGGL((stack_embed_kernel<bf16_t, S>), dim3(M), dim3(ROW_THREADS), 0, s, idx, (const bf16_t*)embed, scale, step, vocab, x, \
                            x0, norm, norm_w, eps, (bf16_t*)h, width, width_p)
    STEPS_SWITCH(width_p, CALL);
#undef CALL
    NC_CHECK_LAUNCH("stack_embed");
    return 0;
}

int nc_launch_stack_row_add(int dtype, const NcRowAdd& a, float eps, int M, int n_rows, int width, int width_p, hipStream_t s) {
    NC_CHECK_ARG(width_p % 4 == 0 && width <= width_p && width_p <= 8192, "stack_row_add: width %d", width_p);
    if (n_rows == 0) return 0;
    NcProfScope prof(NC_CLS_ROWS, (double)n_rows * width_p * (8 + (dtype ? 4 : 2) + 4.0 * (a.partials ? a.splits : 0) + (a.expert_out ? 2.0 * a.top : 0)), s);
#define CALL(S)                                                                                                                  \
    if (dtype) hipLaunchKernelGGL((stack_row_add_kernel<float, S>), dim3(n_rows), dim3(ROW_THREADS), 0, s, a, eps, M, width, width_p); \
    else hipLaunchKernelGGL((stack_row_add_kernel<bf16_t, S>), dim3(n_rows), dim3(ROW_THREADS), 0, s, a, eps, M, width, width_p)
    STEPS_SWITCH(width_p, CALL);
#undef CALL
    NC_CHECK_LAUNCH("stack_row_add");
    return 0;
}

int nc_launch_stack_route(const NcRoute& r, int M, hipStream_t s) {
    NC_CHECK_ARG(r.experts >= 1 && r.experts <= ROUTE_MAX_EXPERTS && r.top >= 1 && r.top <= 64 && r.top <= r.experts, "route: %d of %d experts", r.top,
                 r.experts);
    NcProfScope prof(NC_CLS_ROWS, (double)M * r.experts * 4, s);
    if (M <= 64) {
        hipLaunchKernelGGL((route_sort_kernel<true>), dim3(1), dim3(1024), 0, s, r, M);
    } else {
        hipLaunchKernelGGL(route_choose_kernel, dim3((M + 3) / 4), dim3(256), 0, s, r, M);
        hipLaunchKernelGGL((route_sort_kernel<false>), dim3(1), dim3(1024), 0, s, r, M);
    }
    NC_CHECK_LAUNCH("route");
    return 0;
}

int nc_launch_stack_cache_copy(const void* src, void* dst, int src_rows, int dst_rows, int64_t src_stride, int64_t dst_stride, int64_t bytes,
                               hipStream_t s) {
    NC_CHECK_ARG(src && dst && (src_rows == 1 || src_rows == dst_rows) && dst_rows > 0, "stack_cache_copy: bad rows");
    NC_CHECK_ARG(bytes % 16 == 0 && src_stride % 16 == 0 && dst_stride % 16 == 0, "stack_cache_copy: sizes must be multiples of 16 bytes");
    if (bytes == 0) return 0;
    NcProfScope prof(NC_CLS_ROWS, 2.0 * bytes * dst_rows, s);
    const int64_t pieces = bytes / 16;
    const int gx = (int)(pieces / 1024 < 1 ? 1 : pieces / 1024 > 512 ? 512 : pieces / 1024);
    hipLaunchKernelGGL(stack_cache_copy_kernel, dim3(gx, dst_rows), dim3(256), 0, s, (const uint8_t*)src, (uint8_t*)dst, src_rows, src_stride, dst_stride,
                       pieces);
    NC_CHECK_LAUNCH("stack_cache_copy");
    return 0;
}

int nc_launch_joint_gate(int dtype, const float* raw, int cols, int count, const void* gate, int ldg, const float* w, float eps, float scale, void* out,
                         int ldo, int M, hipStream_t s) {
    NC_CHECK_ARG(raw && gate && w && out && cols % 4 == 0 && count > 0 && count <= cols && ldg % 4 == 0 && ldo % 4 == 0, "joint_gate: %d of %d columns", count, cols);
    NcProfScope prof(NC_CLS_ROWS, (double)M * cols * (dtype ? 12 : 8), s);
    if (dtype)
        hipLaunchKernelGGL((joint_gate_kernel<float>), dim3(M), dim3(256), 0, s, raw, cols, count, (const float*)gate, ldg, w, eps, scale, (float*)out, ldo);
    else
        hipLaunchKernelGGL((joint_gate_kernel<bf16_t>), dim3(M), dim3(256), 0, s, raw, cols, count, (const bf16_t*)gate, ldg, w, eps, scale, (bf16_t*)out, ldo);
    NC_CHECK_LAUNCH("joint_gate");
    return 0;
}
