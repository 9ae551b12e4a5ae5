// Latent attention: all heads' keys and values are linear in one cached vector per token, the latent c (rank values, RMS-normed), and the
// heads share one rotated key part k_r.  A cached row is [c | k_r].
//
//     score(i, j, head) = (q_n . W_uk c_j + q_r . k_r,j) * scale         out(i, head) = W_uv sum_j p_ij c_j,   j <= i
//
// Two forms of the same sum:
//   latent space     W_uk is moved to the query (q_n W_uk, one small product per head), the sum over keys runs on the cached rows
//                    themselves, which are then key AND value of every head, and W_uv is applied to its result.  A key costs rank + rot
//                    values whatever the number of heads: the form for few query rows (decode, short portions).
//   expanded         keys and values of every head are made from the cached latents first (one product), then ordinary causal attention:
//                    the form for many query rows, where dim + rot + vdim per key and head is less work than 2 rank + rot.
// Scores, softmax and sums are fp32.  Where the weights meet the bf16 values on the matrix cores they go in as two bf16 terms (the
// rounded weight and what rounding left), so that the product sees them to 16 bits.
#include <atomic>
#include "nc_stack.h"

typedef __bf16 v8bf __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
typedef short v4s __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) v4s* lds_v4s_t;
typedef __attribute__((address_space(3))) uint8_t* lds_u8_t;

#define LA_MASKED (-1.0e30f)   // score (log2 units) of a key the query does not see
#define LA_M_FLOOR (-1.0e20f)  // running maximum before any visible key: far above LA_MASKED, far below any score
#define LA_LAZY 6.0f           // log2 units the running maximum may lag behind before the sums are rescaled
#define LOG2E 1.4426950408889634f

namespace {
__device__ __forceinline__ v8bf as_v8bf(uint4 v) { return __builtin_bit_cast(v8bf, v); }
__device__ __forceinline__ void split_bf16(float p, __bf16& hi, __bf16& lo) {
    hi = (__bf16)p;
    lo = (__bf16)(p - (float)hi);
}
// eight keys of one column out of LDS rows `pitch` bytes apart: the transposing read hands lane i of a 16-lane group element d = i of
// the four keys its lanes point at
__device__ __forceinline__ v8bf tr_read8(lds_u8_t p, int second) {
    const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)p);
    const v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)(p + second));
    return __builtin_bit_cast(v8bf, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// ------------------------------------------------------------------------------------------------ new tokens
// One workgroup per token: its latent (normed) and shared key part (rotated) into the cache, its queries' rotated parts in place or into
// the latent-space queries.
template <typename T>
__global__ __launch_bounds__(128) void latent_append_kernel(NcLatentGeom g, T* __restrict__ proj, int ldp, const float* __restrict__ norm_w, float eps,
                                                            const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                            T* __restrict__ cache, T* __restrict__ q_lat) {
    __shared__ float red[2];
    const int64_t m = blockIdx.x;
    const int b = (int)(m / g.T), t = (int)(m % g.T), pos = seqlens[b] + t;
    const int half = g.rot_dims / 2, qd = g.dim_p + g.rot_p, rw = g.rank_p + g.rot_p;
    T* row = proj + m * ldp;
    const T* kv = row + g.heads * qd;
    const float2* turn = (const float2*)rope + (int64_t)min(pos, rope_len - 1) * half;
    float ss = 0.f;
    for (int j = threadIdx.x; j < g.rank_p; j += 128) {
        const float v = ld_f32(kv + j);
        ss = fmaf(v, v, ss);
    }
    ss = block_sum<2>(ss, red);
    if (pos < g.Tmax) {
        T* crow = cache + ((int64_t)b * g.Tmax + pos) * rw;
        const float inv = 1.0f / sqrtf(ss / (float)g.rank + eps);
        for (int j = threadIdx.x; j < g.rank_p; j += 128) st_f32(crow + j, ld_f32(kv + j) * inv * norm_w[j]);
        const T* kr = kv + g.rank_p;
        for (int i = threadIdx.x; i < g.rot_p; i += 128) {
            float y = ld_f32(kr + i);
            if (i < half) y = y * turn[i].x - ld_f32(kr + i + half) * turn[i].y;
            else if (i < 2 * half) y = y * turn[i - half].x + ld_f32(kr + i - half) * turn[i - half].y;
            st_f32(crow + g.rank_p + i, y);
        }
    }
    // a thread owns a pair (or two dimensions that pass), so turning in place needs no ordering
    const int rest = g.rot_p - 2 * half, units = half + rest;
    for (int u = threadIdx.x; u < g.heads * units; u += 128) {
        const int h = u / units, i = u % units;
        T* q = row + h * qd + g.dim_p;
        T* o = q_lat ? q_lat + (m * g.heads + h) * rw + g.rank_p : q;
        if (i < half) {
            const float a = ld_f32(q + i), c = ld_f32(q + i + half);
            st_f32(o + i, a * turn[i].x - c * turn[i].y);
            st_f32(o + i + half, c * turn[i].x + a * turn[i].y);
        } else {
            st_f32(o + i + half, ld_f32(q + i + half));
        }
    }
}

// ------------------------------------------------------------------------------------------------ latent space, plain
// One workgroup per query row, any sizes, either storage type: the 32-bit path, and bf16 sizes the matrix-core kernel does not take.
constexpr int SIMPLE_COLS = 16;      // columns of the latent per thread: rank_p <= 256 * 16
template <typename T>
__global__ __launch_bounds__(256) void latent_simple_kernel(NcLatentGeom g, const T* __restrict__ q_lat, const T* __restrict__ cache,
                                                            const int32_t* __restrict__ seqlens, T* __restrict__ out) {
    extern __shared__ float qs[];                 // the query, then 256 weights
    __shared__ float red[4];
    const int rw = g.rank_p + g.rot_p;
    float* const ps = qs + rw;
    const int64_t row = blockIdx.x;
    const int b = (int)(row / ((int64_t)g.T * g.heads)), t = (int)(row / g.heads % g.T);
    const int last = min(seqlens[b] + t, g.Tmax - 1);
    for (int i = threadIdx.x; i < rw; i += 256) qs[i] = ld_f32(q_lat + row * rw + i);
    __syncthreads();
    const T* keys = cache + (int64_t)b * g.Tmax * rw;
    float acc[SIMPLE_COLS];
#pragma unroll
    for (int i = 0; i < SIMPLE_COLS; i++) acc[i] = 0.f;
    float m_run = LA_M_FLOOR, l_run = 0.f;
    for (int k0 = 0; k0 <= last; k0 += 256) {
        const int key = k0 + threadIdx.x, n = min(256, last + 1 - k0);
        float s = LA_MASKED;
        if (key <= last) {
            const T* kr = keys + (int64_t)key * rw;
            v4f d = v4f{0.f, 0.f, 0.f, 0.f};
            for (int i = 0; i < rw; i += 4) {
                const v4f kv = ld4_f32(kr + i);
                d[0] = fmaf(kv[0], qs[i], d[0]), d[1] = fmaf(kv[1], qs[i + 1], d[1]);
                d[2] = fmaf(kv[2], qs[i + 2], d[2]), d[3] = fmaf(kv[3], qs[i + 3], d[3]);
            }
            s = ((d[0] + d[1]) + (d[2] + d[3])) * g.scale;
        }
        float mx = wave_max(s);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float m_new = fmaxf(m_run, mx), corr = expf(m_run - m_new);
        const float p = key <= last ? expf(s - m_new) : 0.f;
        ps[threadIdx.x] = p;
        const float sum = block_sum<4>(p, red);          // (its barriers also order ps)
        l_run = l_run * corr + sum;
        m_run = m_new;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < SIMPLE_COLS; i++) {
            const int c = threadIdx.x + 256 * i;
            if (c >= g.rank_p) break;
            float a = acc[i] * corr;
            for (int j = 0; j < n; j++) a = fmaf(ps[j], ld_f32(keys + (int64_t)(k0 + j) * rw + c), a);
            acc[i] = a;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < SIMPLE_COLS; i++) {
        const int c = threadIdx.x + 256 * i;
        if (c >= g.rank_p) break;
        st_f32(out + row * g.rank_p + c, acc[i] / l_run);
    }
}

// ------------------------------------------------------------------------------------------------ latent space, matrix cores
// A workgroup of eight waves takes 16 query rows (row = token * heads + head of one batch row) and a share of the keys, 32 keys at a time
// through LDS:
//   scores   wave w multiplies keys 16 (w % 2) .. + 15 with all 16 queries over one quarter of the row (S^T = K Q^T), sums into LDS;
//   softmax  wave w takes queries 2 w and 2 w + 1 (32 lanes each, lane = key): running maximum, weights as two bf16 terms and the factor
//            of the sums so far into LDS;
//   sums     wave w adds the columns 16 (w + 8 n) .. + 15 of the latent: O^T += C^T P^T, C^T through the transposing LDS read.
// The rows of the next 32 keys are in flight in registers meanwhile, and two workgroups share a compute unit: a block is a chain of short
// phases with a barrier behind each, and one workgroup works while the other waits.
constexpr int KEYS = 32, SB_PITCH = KEYS + 4, P_PITCH = KEYS * 2 + 16, MFMA_WAVES = 8, MFMA_THREADS = 64 * MFMA_WAVES;
constexpr int MFMA_SMALL_LDS = 4 * 16 * SB_PITCH * 4 + 2 * 16 * P_PITCH + 2 * 16 * 4;      // scores, weights, factors and sums
template <int NT, int PC>
__global__ __launch_bounds__(MFMA_THREADS) void latent_mfma_kernel(NcLatentGeom g, const bf16_t* __restrict__ q_lat, const bf16_t* __restrict__ cache,
                                                                   const int32_t* __restrict__ seqlens, bf16_t* __restrict__ out,
                                                                   float* __restrict__ partials, int splits, int groups) {
    extern __shared__ __align__(16) uint8_t lds[];
    const int rw = g.rank_p + g.rot_p, pitch = rw * 2 + 16, pieces = rw / 32;
    uint8_t* const lds_q = lds + KEYS * pitch;
    float* const sb = (float*)(lds_q + 16 * pitch);                                    // [quarter of the row][query][key]
    uint8_t* const pb = (uint8_t*)(sb + 4 * 16 * SB_PITCH);                            // [hi, lo][query][key] bf16
    float* const factor = (float*)(pb + 2 * 16 * P_PITCH);                             // [query]: of the sums so far
    float* const sums = factor + 16;                                                   // [query]: of the weights, at the end
    // workgroups that read the same keys for other query rows follow each other on one XCD (dealt in turn by the linear index), so that
    // the keys come out of its L2 the second time
    const int slot = (int)blockIdx.x >> 3, group = slot % groups, unit = slot / groups * 8 + ((int)blockIdx.x & 7);
    const int b = unit / splits, split = unit % splits;
    if (b >= g.B) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int col = lane & 15, quad = lane >> 4, ktile = wave & 1, quarter = wave >> 1;
    const int rows = g.T * g.heads, r0 = group * 16;
    const int pos0 = seqlens[b];
    const int per = ((g.pos_max + g.T + KEYS - 1) / KEYS + splits - 1) / splits * KEYS;
    const int k_begin = split * per;
    const int k_end = min(min(k_begin + per, pos0 + min(r0 + 15, rows - 1) / g.heads + 1), g.Tmax);      // exclusive
    const bf16_t* const keys = cache + (int64_t)b * g.Tmax * rw;
    const float scale2 = g.scale * LOG2E;

    // 32 cached rows are one contiguous run of memory, 512 pieces of 16 bytes at a time; `put` is where this thread's pieces go in LDS
    const int total = KEYS * 4 * pieces;
    uint4 rk[PC];
    int put[PC];
#pragma unroll
    for (int i = 0; i < PC; i++) {
        const int idx = tid + MFMA_THREADS * i;
        put[i] = idx < total ? idx / (4 * pieces) * pitch + idx % (4 * pieces) * 16 : -1;
    }
    auto fetch = [&](int kb) {
        const bf16_t* src = keys + (int64_t)kb * rw;
        const int last = (k_end - kb) * 4 * pieces - 1;          // pieces past the last key re-read its last one (weight zero)
#pragma unroll
        for (int i = 0; i < PC; i++)
            if (MFMA_THREADS * i < total) {
                const bf16_t* piece = src + min(tid + MFMA_THREADS * i, last) * 8;
                rk[i] = groups == 1 ? nt_load16(piece) : *(const uint4*)piece;
            }
    };
    if (k_begin < k_end) fetch(k_begin);
    {   // the queries: thread = (row, piece of 16 bytes)
        const int qr = tid >> 5, qp = tid & 31;
        const bf16_t* src = q_lat + ((int64_t)b * rows + min(r0 + qr, rows - 1)) * rw;
        for (int c = qp; c < rw / 8; c += 32) *(uint4*)(lds_q + qr * pitch + c * 16) = *(const uint4*)(src + c * 8);
    }
    v4f acc[NT];
#pragma unroll
    for (int n = 0; n < NT; n++) acc[n] = v4f{0.f, 0.f, 0.f, 0.f};
    // softmax: this lane's query row, its last visible key, and its key of a block
    const int srow = 2 * wave + (lane >> 5), skey = lane & 31;
    const int limit = pos0 + min(r0 + srow, rows - 1) / g.heads;
    float m_run = LA_M_FLOOR, l_run = 0.f;
    const int ntiles = g.rank_p / 16;
    const lds_u8_t tr = (lds_u8_t)lds + (8 * quad + (col >> 2)) * pitch + (16 * wave + 4 * (lane & 3)) * 2;
    const int c_begin = pieces * quarter / 4, c_end = pieces * (quarter + 1) / 4;
    const uint8_t* const kp = lds + (16 * ktile + col) * pitch + quad * 16;
    const uint8_t* const qp = lds_q + col * pitch + quad * 16;

    for (int kb = k_begin; kb < k_end; kb += KEYS) {
        __syncthreads();                    // everyone is done with the previous keys and weights
#pragma unroll
        for (int i = 0; i < PC; i++)
            if (MFMA_THREADS * i < total && put[i] >= 0) *(uint4*)(lds + put[i]) = rk[i];
        __syncthreads();
        if (kb + KEYS < k_end) fetch(kb + KEYS);
        v4f s[2] = {v4f{0.f, 0.f, 0.f, 0.f}, v4f{0.f, 0.f, 0.f, 0.f}};
        int c = c_begin;
        for (; c + 4 <= c_end; c += 4) {
            v8bf kf[4], qf[4];
#pragma unroll
            for (int u = 0; u < 4; u++) kf[u] = as_v8bf(*(const uint4*)(kp + (c + u) * 64)), qf[u] = as_v8bf(*(const uint4*)(qp + (c + u) * 64));
#pragma unroll
            for (int u = 0; u < 4; u++) s[u & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[u], qf[u], s[u & 1], 0, 0, 0);
        }
        for (; c < c_end; c++)
            s[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_v8bf(*(const uint4*)(kp + c * 64)), as_v8bf(*(const uint4*)(qp + c * 64)), s[0], 0, 0, 0);
        *(v4f*)(sb + (16 * quarter + col) * SB_PITCH + 16 * ktile + 4 * quad) = (s[0] + s[1]) * scale2;
        __syncthreads();
        {
            const float* sp = sb + srow * SB_PITCH + skey;
            const float sum = (sp[0] + sp[16 * SB_PITCH]) + (sp[32 * SB_PITCH] + sp[48 * SB_PITCH]);
            const float sc = kb + skey <= min(limit, k_end - 1) ? sum : LA_MASKED;
            float mx = sc;
            mx = fmaxf(mx, dpp_f32<0x128>(mx));
            mx = fmaxf(mx, dpp_f32<0x124>(mx));
            mx = fmaxf(mx, dpp_f32<0x122>(mx));
            mx = fmaxf(mx, dpp_f32<0x121>(mx));
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            const float m_new = fmaxf(m_run, mx), corr = __builtin_amdgcn_exp2f(m_run - m_new);
            const float w = __builtin_amdgcn_exp2f(sc - m_new);
            m_run = m_new;
            l_run = l_run * corr + w;
            const bf16_t hi = f32_to_bf16(w);
            *(bf16_t*)(pb + srow * P_PITCH + skey * 2) = hi;
            *(bf16_t*)(pb + (16 + srow) * P_PITCH + skey * 2) = f32_to_bf16(w - bf16_to_f32(hi));
            if ((lane & 31) == 0) factor[srow] = corr;
        }
        __syncthreads();
        const float corr = factor[col];
        const v8bf hi = as_v8bf(*(const uint4*)(pb + col * P_PITCH + 16 * quad)), lo = as_v8bf(*(const uint4*)(pb + (16 + col) * P_PITCH + 16 * quad));
#pragma unroll
        for (int n = 0; n < NT; n++)
            if (wave + MFMA_WAVES * n < ntiles) {
                const v8bf c0 = tr_read8(tr + 256 * n, 4 * pitch);
                acc[n] *= corr;
                acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c0, hi, acc[n], 0, 0, 0);
                acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c0, lo, acc[n], 0, 0, 0);
            }
    }
    l_run = row16_sum(l_run);
    l_run += __shfl_xor(l_run, 16);
    if ((lane & 31) == 0) {
        sums[srow] = l_run;
        if (splits > 1 && r0 + srow < rows) {
            float* part = partials + (((int64_t)b * rows + r0 + srow) * splits + split) * (g.rank_p + 4);
            part[0] = m_run, part[1] = l_run;
        }
    }
    __syncthreads();
    if (r0 + col >= rows) return;
    const int64_t row = (int64_t)b * rows + r0 + col;
    const float inv = sums[col] > 0.f ? 1.0f / sums[col] : 0.f;
    float* part = partials + (row * splits + split) * (g.rank_p + 4) + 4;
#pragma unroll
    for (int n = 0; n < NT; n++)
        if (wave + MFMA_WAVES * n < ntiles) {
            const int c = 16 * (wave + MFMA_WAVES * n) + 4 * quad;
            if (splits == 1) st4_f32(out + row * g.rank_p + c, acc[n] * inv);
            else *(v4f*)(part + c) = acc[n];
        }
}

constexpr int MAX_SPLITS = 32;
__global__ __launch_bounds__(128) void latent_combine_kernel(const float* __restrict__ partials, int splits, int rank_p, bf16_t* __restrict__ out) {
    __shared__ float weight[64];
    const int64_t row = blockIdx.x;
    const int stride = rank_p + 4;
    const float* part = partials + row * splits * stride;
    if (threadIdx.x < 64) {                     // lane = split (MAX_SPLITS <= 64)
        const bool in = (int)threadIdx.x < splits;
        const float m = in ? part[(int64_t)threadIdx.x * stride] : LA_M_FLOOR, l = in ? part[(int64_t)threadIdx.x * stride + 1] : 0.f;
        const float w = __builtin_amdgcn_exp2f(m - wave_max(m));
        const float total = wave_sum(l * w);
        weight[threadIdx.x] = total > 0.f ? w / total : 0.f;
    }
    __syncthreads();
    for (int c = 4 * threadIdx.x; c < rank_p; c += 512) {
        v4f a = v4f{0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < splits; s0 += 8) {
            v4f p[8];
#pragma unroll
            for (int s = 0; s < 8; s++) p[s] = *(const v4f*)(part + (int64_t)min(s0 + s, splits - 1) * stride + 4 + c);
#pragma unroll
            for (int s = 0; s < 8; s++)
                if (s0 + s < splits) a += p[s] * weight[s0 + s];
        }
        st4_f32(out + row * rank_p + c, a);
    }
}

// ------------------------------------------------------------------------------------------------ expanded
// Causal flash attention forward, written transposed so that nothing moves between lanes (S^T = K Q^T, O^T = V^T P^T with
// v_mfma_f32_32x32x16_bf16; a lane owns one query's column of both): NW waves of 32 queries each, one head per workgroup, 16 NW keys at a
// time through LDS.  A key's row is its head's unrotated part (from kv, up to DN values) and the shared rotated part (from the cache, up to
// DR); keys and values come through buffer descriptors that end behind the workgroup's last key, pieces past a head's own sizes through
// an offset no descriptor reaches: both read zeros.
#define LA_OOB 0x80000000u
template <int DN, int DR, int DV, int NW>
__global__ __launch_bounds__(64 * NW) __attribute__((amdgpu_waves_per_eu(2, 2))) void latent_expanded_kernel(
    NcLatentGeom g, const bf16_t* __restrict__ q, int ldq, const bf16_t* __restrict__ kv, int keys_alloc, const bf16_t* __restrict__ cache,
    const int32_t* __restrict__ seqlens, bf16_t* __restrict__ out, int ldo) {
    constexpr int DQK = DN + DR, KPITCH = DQK * 2 + 16, VPITCH = DV * 2 + 64, NTHR = 64 * NW, KB = 16 * NW, QT = 32 * NW;
    constexpr int NCH = DN / 8, RCH = DR / 8, VCH = DV / 8, NL = KB * NCH / NTHR, RL = KB * RCH / NTHR, VL = KB * VCH / NTHR;
    __shared__ __align__(16) uint8_t lds[KB * KPITCH + KB * VPITCH];
    uint8_t* const lds_v = lds + KB * KPITCH;
    const lds_u8_t lds_v3 = (lds_u8_t)lds + KB * KPITCH;
    const int b = blockIdx.z;
    int h, qb0;
    {   // XCD x gets a contiguous run of (head, tile) units, within a head the longest tiles first
        const int nx = gridDim.x, total = nx * (int)gridDim.y, lid = (int)blockIdx.x + nx * (int)blockIdx.y;
        const int xcd = lid & 7, unit = xcd * (total >> 3) + min(xcd, total & 7) + (lid >> 3);
        h = unit / nx;
        qb0 = (nx - 1 - unit % nx) * QT;
    }
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int col = lane & 31, hl = lane >> 5;
    const int qw0 = qb0 + 32 * wave, t = qw0 + col;
    const bool q_ok = t < g.T;
    const int pos0 = seqlens[b];
    const int qpos = pos0 + min(t, g.T - 1);
    const int k_hi = min(pos0 + min(qb0 + QT - 1, g.T - 1), keys_alloc - 1);
    const int w_hi = pos0 + min(qw0 + 31, g.T - 1), f_hi = min(pos0 + min(qw0, g.T - 1), k_hi);      // seen by some / by all queries of the wave
    const int qd = g.dim_p + g.rot_p, head_w = g.dim_p + g.vdim_p, rw = g.rank_p + g.rot_p;

    v8bf qf[DQK / 16];
    {
        const bf16_t* qrow = q + ((int64_t)b * g.T + min(t, g.T - 1)) * ldq + h * qd;
#pragma unroll
        for (int c = 0; c < DQK / 16; c++) {
            // unrotated dimensions in columns [0, DN), rotated ones from DN on
            const int d = 16 * c + 8 * hl, at = d < DN ? d : g.dim_p + (d - DN);
            const bool in = d < DN ? d < g.dim_p : d - DN < g.rot_p;
            qf[c] = as_v8bf(in ? *(const uint4*)(qrow + at) : make_uint4(0, 0, 0, 0));
        }
    }
    v16f o[DV / 32];
#pragma unroll
    for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[dt][r] = 0.f;
    float m_run = LA_M_FLOOR, l_run = 0.f;
    const float sc = g.scale * LOG2E;

    // staging: 16-byte piece idx = tid + NTHR i of the block's keys
    typedef int ld_v4i __attribute__((ext_vector_type(4)));
    const uint32_t kv_stride = (uint32_t)g.heads * head_w * 2, rot_stride = (uint32_t)rw * 2;
    const __amdgpu_buffer_rsrc_t desc_kv = __builtin_amdgcn_make_buffer_rsrc((void*)(kv + (int64_t)b * keys_alloc * g.heads * head_w + h * head_w), 0,
                                                                             (uint32_t)k_hi * kv_stride + head_w * 2, 0x00020000);
    const __amdgpu_buffer_rsrc_t desc_rot = __builtin_amdgcn_make_buffer_rsrc((void*)(cache + (int64_t)b * g.Tmax * rw + g.rank_p), 0,
                                                                              (uint32_t)k_hi * rot_stride + g.rot_p * 2, 0x00020000);
    uint32_t off_n[NL], off_r[RL], off_v[VL];
#pragma unroll
    for (int i = 0; i < NL; i++) {
        const int idx = tid + NTHR * i, d = 8 * (idx % NCH);
        off_n[i] = d < g.dim_p ? (uint32_t)(idx / NCH) * kv_stride + d * 2 : LA_OOB;
    }
#pragma unroll
    for (int i = 0; i < RL; i++) {
        const int idx = tid + NTHR * i, d = 8 * (idx % RCH);
        off_r[i] = d < g.rot_p ? (uint32_t)(idx / RCH) * rot_stride + d * 2 : LA_OOB;
    }
#pragma unroll
    for (int i = 0; i < VL; i++) {
        const int idx = tid + NTHR * i, d = 8 * (idx % VCH);
        off_v[i] = d < g.vdim_p ? (uint32_t)(idx / VCH) * kv_stride + (g.dim_p + d) * 2 : LA_OOB;
    }
    ld_v4i rn[NL], rr[RL], rv[VL];
    // (the offset of the block is added only to offsets inside the buffers: an LA_OOB one stays where it is)
    auto fetch = [&](int kb) {
        const uint32_t bk = (uint32_t)kb * kv_stride, br = (uint32_t)kb * rot_stride;
#pragma unroll
        for (int i = 0; i < NL; i++) rn[i] = __builtin_amdgcn_raw_buffer_load_b128(desc_kv, off_n[i] == LA_OOB ? LA_OOB : off_n[i] + bk, 0, 0);
#pragma unroll
        for (int i = 0; i < RL; i++) rr[i] = __builtin_amdgcn_raw_buffer_load_b128(desc_rot, off_r[i] == LA_OOB ? LA_OOB : off_r[i] + br, 0, 0);
#pragma unroll
        for (int i = 0; i < VL; i++) rv[i] = __builtin_amdgcn_raw_buffer_load_b128(desc_kv, off_v[i] == LA_OOB ? LA_OOB : off_v[i] + bk, 0, 0);
    };
    auto stage = [&]() {
#pragma unroll
        for (int i = 0; i < NL; i++) {
            const int idx = tid + NTHR * i;
            *(ld_v4i*)(lds + (idx / NCH) * KPITCH + (idx % NCH) * 16) = rn[i];
        }
#pragma unroll
        for (int i = 0; i < RL; i++) {
            const int idx = tid + NTHR * i;
            *(ld_v4i*)(lds + (idx / RCH) * KPITCH + DN * 2 + (idx % RCH) * 16) = rr[i];
        }
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int idx = tid + NTHR * i;
            *(ld_v4i*)(lds_v + (idx / VCH) * VPITCH + (idx % VCH) * 16) = rv[i];
        }
    };
    const uint32_t vtr = (uint32_t)(4 * hl + ((lane & 15) >> 2)) * VPITCH + (16 * ((lane >> 4) & 1) + 4 * (lane & 3)) * 2;
    auto sub_block = [&](int kb, int sb, bool masked) {
        v16f s;
#pragma unroll
        for (int r = 0; r < 16; r++) s[r] = 0.f;
        const uint8_t* kt = lds + (32 * sb + col) * KPITCH + 16 * hl;
#pragma unroll
        for (int c = 0; c < DQK / 16; c++) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(as_v8bf(*(const uint4*)(kt + 32 * c)), qf[c], s, 0, 0, 0);
        if (masked) {                      // wave-uniform
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int key = kb + 8 * (r >> 2) + 4 * hl + (r & 3);
                s[r] = key <= qpos && key <= k_hi ? s[r] * sc : LA_MASKED;
            }
        } else {
#pragma unroll
            for (int r = 0; r < 16; r++) s[r] *= sc;
        }
        float mx = s[0];
#pragma unroll
        for (int r = 1; r < 16; r++) mx = fmaxf(mx, s[r]);
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float m_new = fmaxf(m_run, mx);
        if (__builtin_amdgcn_ballot_w64(m_new > m_run + LA_LAZY) != 0) {      // wave-uniform
            const float corr = __builtin_amdgcn_exp2f(m_run - m_new);
            l_run *= corr;
#pragma unroll
            for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
                for (int r = 0; r < 16; r++) o[dt][r] *= corr;
            m_run = m_new;
        }
        v8bf hi[2], lo[2];
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const float p = __builtin_amdgcn_exp2f(s[r] - m_run);
            l_run += p;
            __bf16 ph, pl;
            split_bf16(p, ph, pl);
            hi[r >> 3][r & 7] = ph, lo[r >> 3][r & 7] = pl;
        }
#pragma unroll
        for (int c2 = 0; c2 < 2; c2++)
#pragma unroll
            for (int dt = 0; dt < DV / 32; dt++) {
                const v8bf vf = tr_read8(lds_v3 + (32 * sb + 16 * c2) * VPITCH + vtr + 64 * dt, 8 * VPITCH);
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, hi[c2], o[dt], 0, 0, 0);
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, lo[c2], o[dt], 0, 0, 0);
            }
    };
    fetch(0);
    for (int kb = 0; kb <= k_hi; kb += KB) {
        __syncthreads();
        stage();
        __syncthreads();
        if (kb + KB <= k_hi) fetch(kb + KB);
#pragma unroll 1
        for (int sb = 0; sb < KB / 32; sb++) {
            const int k0 = kb + 32 * sb;
            if (k0 <= w_hi) sub_block(k0, sb, k0 + 31 > f_hi);
        }
    }
    const float l_tot = l_run + __shfl_xor(l_run, 32);
    const float inv = l_tot > 0.f ? 1.0f / l_tot : 0.f;
    if (!q_ok) return;
    bf16_t* orow = out + ((int64_t)b * g.T + t) * ldo + h * g.vdim_p;
#pragma unroll
    for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
        for (int g4 = 0; g4 < 4; g4++) {
            const int d = 32 * dt + 8 * g4 + 4 * hl;
            if (d < g.vdim_p) st4_f32(orow + d, v4f{o[dt][4 * g4], o[dt][4 * g4 + 1], o[dt][4 * g4 + 2], o[dt][4 * g4 + 3]} * inv);
        }
}

// ------------------------------------------------------------------------------------------------ launches
// the matrix-core kernel's variant for these sizes (0: none), and how many workgroups share the keys of 16 query rows
int mfma_lds_bytes(const NcLatentGeom& g) {
    const int pitch = (g.rank_p + g.rot_p) * 2 + 16;
    return (KEYS + 16) * pitch + MFMA_SMALL_LDS;
}
int mfma_variant(int dtype, const NcLatentGeom& g) {
    const int pieces = (g.rank_p + g.rot_p) / 32;
    if (dtype != 0 || mfma_lds_bytes(g) > 160 * 1024) return 0;
    if (g.rank_p <= 128 && pieces <= 8) return 1;
    if (g.rank_p <= 256 && pieces <= 12) return 2;
    if (g.rank_p <= 512 && pieces <= 20) return 4;
    return 0;
}
int mfma_splits(const NcLatentGeom& g) {
    const int groups = (g.T * g.heads + 15) / 16, blocks = (g.pos_max + g.T + KEYS - 1) / KEYS;
    // two workgroups per compute unit (what their LDS holds): all of them start and end together.  More than 32 shares cost more to merge
    // than they save (2016 keys, 16 heads: 17 us with 24 or 32 shares of one row's keys, 19 with 64)
    int splits = 2 * nc_cu_count() / (g.B * groups);
    if (splits > blocks) splits = blocks;
    return splits < 1 ? 1 : splits > MAX_SPLITS ? MAX_SPLITS : splits;
}
int reserve_lds(const void* fn, int bytes, std::atomic<uint64_t>& done) {
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev > 63) dev = 0;
    if (bytes <= 64 * 1024 || (done.load(std::memory_order_relaxed) >> dev & 1)) return 0;
    if (hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess)
        NC_FAIL(-2, "latent attention: %d bytes of LDS refused", bytes);
    done.fetch_or(1ull << dev, std::memory_order_relaxed);
    return 0;
}
template <int NT, int PC>
int launch_mfma(const NcLatentGeom& g, const bf16_t* q, const bf16_t* cache, const int32_t* seqlens, bf16_t* out, float* partials, int splits, hipStream_t s) {
    const int groups = (g.T * g.heads + 15) / 16, bytes = mfma_lds_bytes(g);
    static std::atomic<uint64_t> done{0};
    if (int rc = reserve_lds((const void*)latent_mfma_kernel<NT, PC>, bytes, done)) return rc;
    hipLaunchKernelGGL((latent_mfma_kernel<NT, PC>), dim3((splits * g.B + 7) / 8 * 8 * groups), dim3(MFMA_THREADS), bytes, s, g, q, cache, seqlens, out, partials, splits, groups);
    NC_CHECK_LAUNCH("latent_mfma");
    return 0;
}
template <int DN, int DR, int DV>
int launch_expanded(const NcLatentGeom& g, const bf16_t* q, int ldq, const bf16_t* kv, int keys, const bf16_t* cache, const int32_t* seqlens, bf16_t* out,
                    int ldo, hipStream_t s) {
    if ((int64_t)((g.T + 127) / 128) * g.heads * g.B >= 200)
        hipLaunchKernelGGL((latent_expanded_kernel<DN, DR, DV, 4>), dim3((g.T + 127) / 128, g.heads, g.B), dim3(256), 0, s, g, q, ldq, kv, keys, cache,
                           seqlens, out, ldo);
    else
        hipLaunchKernelGGL((latent_expanded_kernel<DN, DR, DV, 2>), dim3((g.T + 63) / 64, g.heads, g.B), dim3(128), 0, s, g, q, ldq, kv, keys, cache, seqlens,
                           out, ldo);
    NC_CHECK_LAUNCH("latent_expanded");
    return 0;
}
}  // namespace

int nc_launch_latent_append(int dtype, const NcLatentGeom& g, void* proj, int ldp, const float* norm_w, float eps, const float* rope, int rope_len,
                            const int32_t* seqlens, void* cache, void* q_lat, hipStream_t s) {
    NC_CHECK_ARG(g.rot_dims % 2 == 0 && g.rot_dims <= g.rot_p && g.rank <= g.rank_p, "latent_append: rot_dims=%d rot_p=%d", g.rot_dims, g.rot_p);
    NC_CHECK_ARG(g.pos_max + g.T <= rope_len, "latent_append: position %d past the rotary table of %d", g.pos_max + g.T, rope_len);
    NcProfScope prof(NC_CLS_ROWS, (double)g.B * g.T * (g.rank_p + g.rot_p * (2.0 + g.heads)) * (dtype ? 8 : 4), s);
    if (dtype)
        hipLaunchKernelGGL((latent_append_kernel<float>), dim3(g.B * g.T), dim3(128), 0, s, g, (float*)proj, ldp, norm_w, eps, rope, rope_len, seqlens,
                           (float*)cache, (float*)q_lat);
    else
        hipLaunchKernelGGL((latent_append_kernel<bf16_t>), dim3(g.B * g.T), dim3(128), 0, s, g, (bf16_t*)proj, ldp, norm_w, eps, rope, rope_len, seqlens,
                           (bf16_t*)cache, (bf16_t*)q_lat);
    NC_CHECK_LAUNCH("latent_append");
    return 0;
}

size_t nc_latent_partial_bytes(int dtype, const NcLatentGeom& g) {
    if (!mfma_variant(dtype, g)) return 0;
    // sized for any cache length the step may see: the split count only falls with it
    const int splits = mfma_splits(g);
    return splits > 1 ? (size_t)g.B * g.T * g.heads * splits * (g.rank_p + 4) * sizeof(float) : 0;
}

int nc_launch_latent_attention(int dtype, const NcLatentGeom& g, const void* q_lat, const void* cache, const int32_t* seqlens, void* out_lat,
                               void* partials, size_t partial_bytes, hipStream_t s) {
    const int rows = g.B * g.T * g.heads;
    // the cached rows are read once per batch row (bytes); what a key costs beyond that stays on the chip
    NcProfScope prof(NC_CLS_LATENT, (double)g.B * (g.pos_max + g.T) * (g.rank_p + g.rot_p) * (dtype ? 4 : 2), s, g.T);
    const int variant = mfma_variant(dtype, g);
    if (variant) {
        const int splits = mfma_splits(g);
        NC_CHECK_ARG(splits == 1 || (partials && partial_bytes >= nc_latent_partial_bytes(dtype, g)), "latent_attention: partial buffer too small");
        const bf16_t *q = (const bf16_t*)q_lat, *c = (const bf16_t*)cache;
        bf16_t* o = (bf16_t*)out_lat;
        float* p = (float*)partials;
        const int rc = variant == 1   ? launch_mfma<1, 2>(g, q, c, seqlens, o, p, splits, s)
                       : variant == 2 ? launch_mfma<2, 3>(g, q, c, seqlens, o, p, splits, s)
                                      : launch_mfma<4, 5>(g, q, c, seqlens, o, p, splits, s);
        if (rc) return rc;
        if (splits > 1) {
            hipLaunchKernelGGL(latent_combine_kernel, dim3(rows), dim3(128), 0, s, p, splits, g.rank_p, o);
            NC_CHECK_LAUNCH("latent_combine");
        }
        return 0;
    }
    NC_CHECK_ARG(g.rank_p <= 256 * SIMPLE_COLS, "latent_attention: a latent of %d values is not supported", g.rank_p);
    const int bytes = (g.rank_p + g.rot_p + 256) * 4;
    if (dtype)
        hipLaunchKernelGGL((latent_simple_kernel<float>), dim3(rows), dim3(256), bytes, s, g, (const float*)q_lat, (const float*)cache, seqlens, (float*)out_lat);
    else
        hipLaunchKernelGGL((latent_simple_kernel<bf16_t>), dim3(rows), dim3(256), bytes, s, g, (const bf16_t*)q_lat, (const bf16_t*)cache, seqlens,
                           (bf16_t*)out_lat);
    NC_CHECK_LAUNCH("latent_simple");
    return 0;
}

bool nc_latent_expanded_ok(int dtype, const NcLatentGeom& g) { return dtype == 0 && g.dim_p <= 128 && g.rot_p <= 64 && g.vdim_p <= 128; }

int nc_launch_latent_expanded(const NcLatentGeom& g, const bf16_t* q, int ldq, const bf16_t* kv, int keys, const bf16_t* cache, const int32_t* seqlens,
                              bf16_t* out, int ldo, hipStream_t s) {
    NC_CHECK_ARG(nc_latent_expanded_ok(0, g) && keys >= g.pos_max + g.T && keys <= g.Tmax, "latent_expanded: sizes not supported");
    const int dqk = g.dim_p + g.rot_p;
    // causal pairs: all earlier keys and half of the new ones
    NcProfScope prof(NC_CLS_LATENT, 2.0 * g.B * g.heads * g.T * (g.pos_max + 0.5 * (g.T + 1)) * (dqk + g.vdim_p), s, g.T);
    NC_CHECK_ARG((int64_t)keys * g.heads * (g.dim_p + g.vdim_p) * 2 < (1ll << 31), "latent_expanded: %d keys past 2 GiB", keys);
#define GO(N, R, V) launch_expanded<N, R, V>(g, q, ldq, kv, keys, cache, seqlens, out, ldo, s)
#define GO_V(N, R) (g.vdim_p <= 64 ? GO(N, R, 64) : GO(N, R, 128))
    if (g.dim_p <= 64) return g.rot_p <= 32 ? GO_V(64, 32) : GO_V(64, 64);
    return g.rot_p <= 32 ? GO_V(128, 32) : GO_V(128, 64);
#undef GO
#undef GO_V
}
