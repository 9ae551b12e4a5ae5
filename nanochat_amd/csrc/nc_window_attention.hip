// Window attention: grouped-query softmax attention in which query i sees the last `window` keys up to itself and, however far away, the
// first `keep_first` of the sequence; a number per head counts in the softmax's denominator without a key or a value (the sink):
//
//     p_ij = exp(s_ij) / (exp(sink) + sum_j' exp(s_ij')),     s_ij = scale (q_i . k_j),     j <= i and (i - j < window or j < keep_first)
//
// q and k are RMS-normed over all heads at once and turned with the position; a cached row is, for every kv head, its normed and turned key
// (dim_p) and its value (vdim_p).
//
// The keys a group of queries may see are two runs: [0, n_keep) and [first, end).  The kernels walk them as one list: entry v is key v
// below n_keep and key v - n_keep + first from there on.  The running maximum starts at the sink and the running sum at exp(0), so the sink
// costs nothing afterwards and a query without any key left in a block needs no special case.
// Scores, softmax and sums are fp32; where the weights meet bf16 values on the matrix cores they go in as two bf16 terms.
//
//   window_few_kernel      decode and short portions: 16 query rows of one kv head, keys dealt to waves and workgroups
//   window_prefill_kernel  long portions: waves of 32 queries of one head, keys through LDS; two waves may share the keys of their queries
//   window_simple_kernel   any sizes, either storage type
#include "nc_stack.h"

typedef __bf16 v8bf __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
typedef short v4s __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) v4s* lds_v4s_t;
typedef __attribute__((address_space(3))) uint8_t* lds_u8_t;

#define WA_MASKED (-1.0e30f)   // score (log2 units) of a key the query does not see
#define WA_M_FLOOR (-1.0e20f)  // running maximum before any visible key: far above WA_MASKED, far below any score
#define WA_LAZY 6.0f           // log2 units the running maximum may lag behind before the sums are rescaled
#define LOG2E 1.4426950408889634f

namespace {
__device__ __forceinline__ v8bf as_v8bf(uint4 v) { return __builtin_bit_cast(v8bf, v); }
__device__ __forceinline__ v8bf tr_read8(lds_u8_t p, int second) {
    const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)p);
    const v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)(p + second));
    return __builtin_bit_cast(v8bf, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// The list of keys that queries at positions [q_lo, q_hi] may see.
struct KeyList {
    int n_keep, first, count;
    __device__ __forceinline__ int key(int v) const { return v < n_keep ? v : v - n_keep + first; }
};
__device__ __forceinline__ KeyList key_list(const NcWindowGeom& g, int q_lo, int q_hi) {
    KeyList l;
    l.n_keep = min(g.keep_first, q_hi + 1);
    l.first = max(q_lo - g.window + 1, l.n_keep);
    l.count = l.n_keep + max(0, q_hi + 1 - l.first);
    return l;
}
__device__ __forceinline__ bool sees(const NcWindowGeom& g, int q, int key) { return key <= q && (q - key < g.window || key < g.keep_first); }

// ------------------------------------------------------------------------------------------------ new tokens
// One workgroup per token.  A thread owns a pair of dimensions that turn together, or two that pass, so turning in place needs no ordering.
template <typename T>
__global__ __launch_bounds__(256) void window_append_kernel(NcWindowGeom g, T* __restrict__ proj, int ldp, const float* __restrict__ bias,
                                                            const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w, float eps,
                                                            const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                            T* __restrict__ cache) {
    __shared__ float red[4];
    const int64_t m = blockIdx.x;
    const int b = (int)(m / g.T), t = (int)(m % g.T), pos = seqlens[b] + t, half = g.rot_dims / 2, rest = g.dim_p - 2 * half;
    const int nq = g.heads * g.dim_p, nk = g.kv_heads * g.dim_p, nv = g.kv_heads * g.vdim_p, head_w = g.dim_p + g.vdim_p;
    T* row = proj + m * ldp;
    const float2* turn = (const float2*)rope + (int64_t)min(pos, rope_len - 1) * half;
    float sq = 0.f, sk = 0.f;
    for (int j = 4 * threadIdx.x; j < nq + nk; j += 1024) {          // (nq is a multiple of 32: four values are all q or all k)
        const v4f v = ld4_f32(row + j) + *(const v4f*)(bias + j);
        const float s = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
        if (j < nq) sq += s;
        else sk += s;
    }
    sq = block_sum<4>(sq, red);
    sk = block_sum<4>(sk, red);
    const float iq = 1.0f / sqrtf(sq / (float)(g.heads * g.dim) + eps), ik = 1.0f / sqrtf(sk / (float)(g.kv_heads * g.dim) + eps);
    const bool in = pos < g.Tmax;
    T* crow = cache + ((int64_t)b * g.Tmax + (in ? pos : 0)) * g.kv_heads * head_w;
    const int units = half + rest;
    for (int u = threadIdx.x; u < (g.heads + g.kv_heads) * units; u += 256) {
        const int h = u / units, i = u % units;
        const bool is_q = h < g.heads;
        if (!is_q && !in) continue;
        const int at = h * g.dim_p;                                  // in the projected row: the k heads follow the q heads
        const float* w = is_q ? q_norm_w + at : k_norm_w + at - nq;
        const float inv = is_q ? iq : ik;
        T* o = is_q ? row + at : crow + (h - g.heads) * head_w;
        if (i < half) {
            const float a = (ld_f32(row + at + i) + bias[at + i]) * inv * w[i], c = (ld_f32(row + at + i + half) + bias[at + i + half]) * inv * w[i + half];
            st_f32(o + i, a * turn[i].x - c * turn[i].y);
            st_f32(o + i + half, c * turn[i].x + a * turn[i].y);
        } else {
            const int d = i + half;
            st_f32(o + d, (ld_f32(row + at + d) + bias[at + d]) * inv * w[d]);
        }
    }
    if (!in) return;
    for (int j = threadIdx.x; j < nv; j += 256) st_f32(crow + j / g.vdim_p * head_w + g.dim_p + j % g.vdim_p, ld_f32(row + nq + nk + j) + bias[nq + nk + j]);
}

// ------------------------------------------------------------------------------------------------ any sizes
// One workgroup per (token, head).
constexpr int SIMPLE_COLS = 4;       // value columns per thread: vdim_p <= 256 * 4
template <typename T>
__global__ __launch_bounds__(256) void window_simple_kernel(NcWindowGeom g, const T* __restrict__ q, int ldq, const T* __restrict__ cache,
                                                            const float* __restrict__ sink, const int32_t* __restrict__ seqlens, T* __restrict__ out, int ldo) {
    extern __shared__ float qs[];                 // the query, then 256 weights
    __shared__ float red[4];
    float* const ps = qs + g.dim_p;
    const int64_t m = blockIdx.x / g.heads;
    const int h = (int)(blockIdx.x % g.heads), kvh = h / (g.heads / g.kv_heads);
    const int b = (int)(m / g.T), pos = min(seqlens[b] + (int)(m % g.T), g.Tmax - 1), head_w = g.dim_p + g.vdim_p, rw = g.kv_heads * head_w;
    const KeyList list = key_list(g, pos, pos);
    for (int i = threadIdx.x; i < g.dim_p; i += 256) qs[i] = ld_f32(q + m * ldq + h * g.dim_p + i);
    __syncthreads();
    const T* keys = cache + (int64_t)b * g.Tmax * rw + kvh * head_w;
    float acc[SIMPLE_COLS];
#pragma unroll
    for (int i = 0; i < SIMPLE_COLS; i++) acc[i] = 0.f;
    float m_run = sink[h], l_run = 1.f;
    for (int v0 = 0; v0 < list.count; v0 += 256) {
        const int v = v0 + threadIdx.x, n = min(256, list.count - v0);
        float s = WA_MASKED;
        if (v < list.count) {
            const T* kr = keys + (int64_t)list.key(v) * rw;
            v4f d = v4f{0.f, 0.f, 0.f, 0.f};
            for (int i = 0; i < g.dim_p; i += 4) {
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
        const float p = v < list.count ? expf(s - m_new) : 0.f;
        ps[threadIdx.x] = p;
        const float sum = block_sum<4>(p, red);          // (its barriers also order ps)
        l_run = l_run * corr + sum;
        m_run = m_new;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < SIMPLE_COLS; i++) {
            const int c = threadIdx.x + 256 * i;
            if (c >= g.vdim_p) break;
            float a = acc[i] * corr;
            for (int j = 0; j < n; j++) a = fmaf(ps[j], ld_f32(keys + (int64_t)list.key(v0 + j) * rw + g.dim_p + c), a);
            acc[i] = a;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < SIMPLE_COLS; i++) {
        const int c = threadIdx.x + 256 * i;
        if (c >= g.vdim_p) break;
        st_f32(out + m * ldo + h * g.vdim_p + c, acc[i] / l_run * g.out_scale);
    }
}

// ------------------------------------------------------------------------------------------------ few query rows
// A workgroup of four waves takes 16 query rows of one kv head (row = token * R + head of the group, R = heads / kv_heads) and a share of
// their keys; a wave takes every fourth block of 32 keys and keeps sums of its own.  Scores S^T = K Q^T: a lane ends up with four keys of one
// query from each half of the block; that is already what the second product O^T = V^T P^T wants, the keys of V being picked in the same
// order by the transposing LDS read, so nothing moves between lanes.  Keys go from memory into the operand registers, values through LDS
// that is the wave's own: no barrier until the waves' sums meet.  The next block is in flight in registers meanwhile.
constexpr int BLOCK_KEYS = 32;
constexpr int MAX_SPLITS = 32;
template <int DQ, int DV>
__global__ __launch_bounds__(256) void window_few_kernel(NcWindowGeom g, const bf16_t* __restrict__ q, int ldq, const bf16_t* __restrict__ cache,
                                                         const float* __restrict__ sink, const int32_t* __restrict__ seqlens, bf16_t* __restrict__ out, int ldo,
                                                         float* __restrict__ partials, int splits, int groups) {
    constexpr int QC = DQ / 32, VP = DV * 2 + 16, VL = DV / 16, NT = DV / 16, V_BYTES = BLOCK_KEYS * VP, O_PITCH = DV + 4;
    constexpr int SUM_BYTES = 4 * 16 * O_PITCH * 4, LDS = 4 * V_BYTES > SUM_BYTES ? 4 * V_BYTES : SUM_BYTES;
    __shared__ __align__(16) uint8_t lds[LDS];
    __shared__ float ms[4][16], ls[4][16];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, quad = lane >> 4;
    const int split = blockIdx.x, group = (int)blockIdx.y % groups, kvh = (int)blockIdx.y / groups, b = blockIdx.z;
    const int R = g.heads / g.kv_heads, rows = g.T * R, r0 = group * 16, r1 = min(r0 + 15, rows - 1);
    const int head_w = g.dim_p + g.vdim_p, rw = g.kv_heads * head_w;
    const int pos0 = min(seqlens[b], g.Tmax - g.T);
    const KeyList list = key_list(g, pos0 + r0 / R, pos0 + r1 / R);
    const int blocks = (list.count + BLOCK_KEYS - 1) / BLOCK_KEYS, per = (blocks + splits - 1) / splits;
    const int b_begin = split * per, b_end = min(blocks, b_begin + per);
    const bf16_t* const keys = cache + (int64_t)b * g.Tmax * rw + kvh * head_w;

    const int row = min(r0 + col, r1), t = row / R, h = kvh * R + row % R, qpos = pos0 + t;
    v8bf qf[QC];
    {
        const bf16_t* src = q + ((int64_t)b * g.T + t) * ldq + h * g.dim_p + 8 * quad;
#pragma unroll
        for (int c = 0; c < QC; c++) qf[c] = as_v8bf(32 * c < g.dim_p ? *(const uint4*)(src + 32 * c) : make_uint4(0, 0, 0, 0));
    }
    const bool has_sink = split == 0 && wave == 0;
    float m_run = has_sink ? sink[h] * LOG2E : WA_M_FLOOR, l_run = has_sink && quad == 0 ? 1.f : 0.f;
    v4f acc[NT];
#pragma unroll
    for (int n = 0; n < NT; n++) acc[n] = v4f{0.f, 0.f, 0.f, 0.f};
    const float scale2 = g.scale * LOG2E;
    uint8_t* const lv = lds + wave * V_BYTES;
    const lds_u8_t tr = (lds_u8_t)lds + wave * V_BYTES + (4 * quad + (col >> 2)) * VP + 4 * (lane & 3) * 2;

    v4i kf[2][QC], vf[VL];
    auto fetch = [&](int blk) {
        const int v0 = blk * BLOCK_KEYS;
#pragma unroll
        for (int s = 0; s < 2; s++) {
            const bf16_t* src = keys + (int64_t)list.key(min(v0 + 16 * s + col, list.count - 1)) * rw + 8 * quad;
#pragma unroll
            for (int c = 0; c < QC; c++)
                kf[s][c] = 32 * c < g.dim_p ? *(const v4i*)(src + 32 * c) : v4i{0, 0, 0, 0};       // uniform
        }
        // values: piece p of 16 bytes is (row p / (DV / 8), columns 8 (p % (DV / 8)) ..)
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int p = lane + 64 * i, r = p / (DV / 8), d = 8 * (p % (DV / 8));
            const bf16_t* src = keys + (int64_t)list.key(min(v0 + r, list.count - 1)) * rw + g.dim_p + min(d, g.vdim_p - 8);
            vf[i] = *(const v4i*)src;
        }
    };
    int blk = b_begin + wave;
    if (blk < b_end) fetch(blk);
    for (; blk < b_end; blk += 4) {
        asm volatile("" ::: "memory");
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int p = lane + 64 * i;
            *(v4i*)(lv + p / (DV / 8) * VP + p % (DV / 8) * 16) = vf[i];
        }
        asm volatile("" ::: "memory");
        __builtin_amdgcn_wave_barrier();
        v4f s[2];
#pragma unroll
        for (int i = 0; i < 2; i++) {
            s[i] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < QC; c++) s[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(v8bf, kf[i][c]), qf[c], s[i], 0, 0, 0);
        }
        if (blk + 4 < b_end) fetch(blk + 4);
        float mx = WA_MASKED;
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int v = blk * BLOCK_KEYS + 16 * i + 4 * quad + r;
                s[i][r] = v < list.count && sees(g, qpos, list.key(v)) ? s[i][r] * scale2 : WA_MASKED;
                mx = fmaxf(mx, s[i][r]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float m_new = fmaxf(m_run, mx);
        if (__builtin_amdgcn_ballot_w64(m_new > m_run + WA_LAZY) != 0) {      // wave-uniform
            const float corr = __builtin_amdgcn_exp2f(m_run - m_new);
            l_run *= corr;
#pragma unroll
            for (int n = 0; n < NT; n++) acc[n] *= corr;
            m_run = m_new;
        }
        v8bf hi, lo;
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const float p = __builtin_amdgcn_exp2f(s[j >> 2][j & 3] - m_run);
            l_run += p;
            hi[j] = (__bf16)p;
            lo[j] = (__bf16)(p - (float)hi[j]);
        }
#pragma unroll
        for (int n = 0; n < NT; n++) {
            const v8bf c0 = tr_read8(tr + 32 * n, 16 * VP);
            acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c0, hi, acc[n], 0, 0, 0);
            acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c0, lo, acc[n], 0, 0, 0);
        }
    }
    l_run += __shfl_xor(l_run, 16);
    l_run += __shfl_xor(l_run, 32);
    __syncthreads();                               // every wave is done with its values
    float* const sums = (float*)lds;
    if (quad == 0) ms[wave][col] = m_run, ls[wave][col] = l_run;
#pragma unroll
    for (int n = 0; n < NT; n++) *(v4f*)(sums + (wave * 16 + col) * O_PITCH + 16 * n + 4 * quad) = acc[n];
    __syncthreads();
    const int qr = tid >> 4, wrow = r0 + qr;
    if (wrow >= rows) return;
    float mt = WA_M_FLOOR, lt = 0.f, f[4];
#pragma unroll
    for (int w = 0; w < 4; w++) mt = fmaxf(mt, ms[w][qr]);
#pragma unroll
    for (int w = 0; w < 4; w++) {
        f[w] = __builtin_amdgcn_exp2f(ms[w][qr] - mt);
        lt += f[w] * ls[w][qr];
    }
    const int64_t orow = (int64_t)b * g.T + wrow / R;
    const int oh = kvh * R + wrow % R;
    float* part = partials + ((orow * g.heads + oh) * splits + split) * (g.vdim_p + 4);
    if (splits > 1 && (tid & 15) == 0) part[0] = mt, part[1] = lt;
    const float inv = lt > 0.f ? g.out_scale / lt : 0.f;
    for (int c = 4 * (tid & 15); c < g.vdim_p; c += 64) {
        v4f y = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 4; w++) y += *(const v4f*)(sums + (w * 16 + qr) * O_PITCH + c) * f[w];
        if (splits > 1) *(v4f*)(part + 4 + c) = y;
        else st4_f32(out + orow * ldo + oh * g.vdim_p + c, y * inv);
    }
}

// One wave per (token, head): lane = split for the weights, then four columns per lane and step.
__global__ __launch_bounds__(64) void window_combine_kernel(const float* __restrict__ partials, int splits, int heads, int vdim_p, float scale,
                                                            bf16_t* __restrict__ out, int ldo) {
    __shared__ float weight[64];
    const int64_t row = blockIdx.x;
    const int stride = vdim_p + 4;
    const float* part = partials + row * splits * stride;
    const bool in = (int)threadIdx.x < splits;
    const float m = in ? part[(int64_t)threadIdx.x * stride] : WA_M_FLOOR, l = in ? part[(int64_t)threadIdx.x * stride + 1] : 0.f;
    const float w = __builtin_amdgcn_exp2f(m - wave_max(m));
    const float total = wave_sum(l * w);
    weight[threadIdx.x] = total > 0.f ? w * scale / total : 0.f;
    __syncthreads();
    for (int c = 4 * threadIdx.x; c < vdim_p; c += 256) {
        v4f a = v4f{0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < splits; s0 += 8) {
            v4f p[8];
#pragma unroll
            for (int s = 0; s < 8; s++) p[s] = *(const v4f*)(part + (int64_t)min(s0 + s, splits - 1) * stride + 4 + c);
#pragma unroll
            for (int s = 0; s < 8; s++)
                if (s0 + s < splits) a += p[s] * weight[s0 + s];
        }
        st4_f32(out + row / heads * ldo + row % heads * vdim_p + c, a);
    }
}

// ------------------------------------------------------------------------------------------------ many query rows
// Flash attention written transposed (S^T = K Q^T, O^T = V^T P^T with v_mfma_f32_32x32x16_bf16; a lane owns one query's column of both):
// NQ groups of 32 queries, one head per workgroup, KB entries of the workgroup's key list at a time through LDS; the blocks of 32 keys are
// dealt to KS waves per group, whose sums meet in LDS at the end.
template <int DQ, int DV, int NQ, int KS>
__global__ __launch_bounds__(64 * NQ * KS) __attribute__((amdgpu_waves_per_eu(2, 2))) void window_prefill_kernel(
    NcWindowGeom g, const bf16_t* __restrict__ q, int ldq, const bf16_t* __restrict__ cache, const float* __restrict__ sink,
    const int32_t* __restrict__ seqlens, bf16_t* __restrict__ out, int ldo) {
    constexpr int KPITCH = DQ * 2 + 16, VPITCH = DV * 2 + 64, NW = NQ * KS, NTHR = 64 * NW, KB = 16 * NW, QT = 32 * NQ;
    constexpr int KCH = DQ / 8, VCH = DV / 8, KL = KB * KCH / NTHR, VL = KB * VCH / NTHR;
    constexpr int STAGE = KB * KPITCH + KB * VPITCH, O_PITCH = DV + 4, SUM = KS > 1 ? NQ * 32 * (O_PITCH + 2) * 4 : 0;
    static_assert(KS == 1 || (KS == 2 && KB >= 64), "every wave has a block of a stage");
    __shared__ __align__(16) uint8_t lds[STAGE > SUM ? STAGE : SUM];
    uint8_t* const lds_v = lds + KB * KPITCH;
    const lds_u8_t lds_v3 = (lds_u8_t)lds + KB * KPITCH;
    const int b = blockIdx.z;
    int h, qb0;
    {   // XCD x gets a contiguous run of (head, tile) units: neighbours read the same keys
        const int nx = gridDim.x, total = nx * (int)gridDim.y, lid = (int)blockIdx.x + nx * (int)blockIdx.y;
        const int xcd = lid & 7, unit = xcd * (total >> 3) + min(xcd, total & 7) + (lid >> 3);
        h = unit / nx;
        qb0 = unit % nx * QT;
    }
    const int kvh = h / (g.heads / g.kv_heads), head_w = g.dim_p + g.vdim_p, rw = g.kv_heads * head_w;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int col = lane & 31, hl = lane >> 5;
    const int qw = wave % NQ, ks = wave / NQ, qw0 = qb0 + 32 * qw, t = qw0 + col;
    const int pos0 = min(seqlens[b], g.Tmax - g.T);
    const int qpos = pos0 + min(t, g.T - 1);
    const int w_lo = pos0 + min(qw0, g.T - 1), w_hi = pos0 + min(qw0 + 31, g.T - 1);
    const KeyList list = key_list(g, pos0 + qb0, pos0 + min(qb0 + QT - 1, g.T - 1));
    const bf16_t* const keys = cache + (int64_t)b * g.Tmax * rw + kvh * head_w;

    v8bf qf[DQ / 16];
    {
        const bf16_t* qrow = q + ((int64_t)b * g.T + min(t, g.T - 1)) * ldq + h * g.dim_p;
#pragma unroll
        for (int c = 0; c < DQ / 16; c++) {
            const int d = 16 * c + 8 * hl;
            qf[c] = as_v8bf(d < g.dim_p ? *(const uint4*)(qrow + d) : make_uint4(0, 0, 0, 0));
        }
    }
    v16f o[DV / 32];
#pragma unroll
    for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[dt][r] = 0.f;
    float m_run = ks == 0 ? sink[h] * LOG2E : WA_M_FLOOR, l_run = ks == 0 && hl == 0 ? 1.f : 0.f;
    const float sc = g.scale * LOG2E;

    // staging: 16-byte piece idx = tid + NTHR i of the block's keys; past a head's own sizes zeros
    uint4 rk[KL], rv[VL];
    auto fetch = [&](int v0) {
#pragma unroll
        for (int i = 0; i < KL; i++) {
            const int idx = tid + NTHR * i, d = 8 * (idx % KCH);
            const bf16_t* src = keys + (int64_t)list.key(min(v0 + idx / KCH, list.count - 1)) * rw;
            rk[i] = d < g.dim_p ? *(const uint4*)(src + d) : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int idx = tid + NTHR * i, d = 8 * (idx % VCH);
            const bf16_t* src = keys + (int64_t)list.key(min(v0 + idx / VCH, list.count - 1)) * rw + g.dim_p;
            rv[i] = d < g.vdim_p ? *(const uint4*)(src + d) : make_uint4(0, 0, 0, 0);
        }
    };
    auto stage = [&]() {
#pragma unroll
        for (int i = 0; i < KL; i++) {
            const int idx = tid + NTHR * i;
            *(uint4*)(lds + (idx / KCH) * KPITCH + (idx % KCH) * 16) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int idx = tid + NTHR * i;
            *(uint4*)(lds_v + (idx / VCH) * VPITCH + (idx % VCH) * 16) = rv[i];
        }
    };
    const uint32_t vtr = (uint32_t)(4 * hl + ((lane & 15) >> 2)) * VPITCH + (16 * ((lane >> 4) & 1) + 4 * (lane & 3)) * 2;
    auto sub_block = [&](int v0, int sb, bool masked) {
        v16f s;
#pragma unroll
        for (int r = 0; r < 16; r++) s[r] = 0.f;
        const uint8_t* kt = lds + (32 * sb + col) * KPITCH + 16 * hl;
#pragma unroll
        for (int c = 0; c < DQ / 16; c++) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(as_v8bf(*(const uint4*)(kt + 32 * c)), qf[c], s, 0, 0, 0);
        if (masked) {                      // wave-uniform
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int v = v0 + 8 * (r >> 2) + 4 * hl + (r & 3);
                s[r] = v < list.count && sees(g, qpos, list.key(v)) ? s[r] * sc : WA_MASKED;
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
        if (__builtin_amdgcn_ballot_w64(m_new > m_run + WA_LAZY) != 0) {      // wave-uniform
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
            hi[r >> 3][r & 7] = (__bf16)p;
            lo[r >> 3][r & 7] = (__bf16)(p - (float)hi[r >> 3][r & 7]);
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
    for (int vb = 0; vb < list.count; vb += KB) {
        __syncthreads();
        stage();
        __syncthreads();
        if (vb + KB < list.count) fetch(vb + KB);
#pragma unroll 1
        for (int sb = ks; sb < KB / 32; sb += KS) {
            const int v0 = vb + 32 * sb;
            if (v0 >= list.count) break;
            // the smallest and largest key of these entries (the list rises), against the wave's queries
            const int k_lo = list.key(v0), k_hi = list.key(min(v0 + 31, list.count - 1));
            if (k_lo > w_hi || (w_lo - k_hi >= g.window && k_lo >= g.keep_first)) continue;            // nobody sees any
            const bool all = v0 + 32 <= list.count && k_hi <= w_lo && (w_hi - k_lo < g.window || k_hi < g.keep_first);
            sub_block(v0, sb, !all);
        }
    }
    l_run += __shfl_xor(l_run, 32);
    if (KS == 2) {
        float* const row = (float*)lds + (32 * qw + col) * (O_PITCH + 2);
        __syncthreads();                       // the last stage has been read
        if (ks == 1) {
            if (hl == 0) row[O_PITCH] = m_run, row[O_PITCH + 1] = l_run;
#pragma unroll
            for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
                for (int r = 0; r < 16; r++) row[32 * dt + 8 * (r >> 2) + 4 * hl + (r & 3)] = o[dt][r];
        }
        __syncthreads();
        if (ks == 1) return;
        const float m2 = row[O_PITCH], mt = fmaxf(m_run, m2), f1 = __builtin_amdgcn_exp2f(m_run - mt), f2 = __builtin_amdgcn_exp2f(m2 - mt);
        l_run = l_run * f1 + row[O_PITCH + 1] * f2;
#pragma unroll
        for (int dt = 0; dt < DV / 32; dt++)
#pragma unroll
            for (int r = 0; r < 16; r++) o[dt][r] = o[dt][r] * f1 + row[32 * dt + 8 * (r >> 2) + 4 * hl + (r & 3)] * f2;
    }
    const float inv = g.out_scale / l_run;
    if (t >= g.T) return;
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
constexpr int PREFILL_MIN_TOKENS = 32;
bool mfma_ok(int dtype, const NcWindowGeom& g) { return dtype == 0 && g.dim_p <= 192 && g.vdim_p <= 128; }
int few_groups(const NcWindowGeom& g) { return (g.T * (g.heads / g.kv_heads) + 15) / 16; }
// workgroups that share the keys of 16 query rows: two per compute unit in all, and no share below one block of keys per wave
int few_splits(const NcWindowGeom& g) {
    const int64_t most = (int64_t)g.window + g.keep_first + g.T;
    const int keys = most < g.pos_max + g.T ? (int)most : g.pos_max + g.T;
    const int by_keys = (keys + 4 * BLOCK_KEYS - 1) / (4 * BLOCK_KEYS);
    int splits = 2 * nc_cu_count() / (g.B * g.kv_heads * few_groups(g));
    if (splits > by_keys) splits = by_keys;
    return splits < 1 ? 1 : splits > MAX_SPLITS ? MAX_SPLITS : splits;
}
bool use_few(const NcWindowGeom& g) { return g.T < PREFILL_MIN_TOKENS; }

template <int DQ, int DV>
int launch_few(const NcWindowGeom& g, const bf16_t* q, int ldq, const bf16_t* cache, const float* sink, const int32_t* seqlens, bf16_t* out, int ldo,
               float* partials, int splits, hipStream_t s) {
    const int groups = few_groups(g);
    hipLaunchKernelGGL((window_few_kernel<DQ, DV>), dim3(splits, groups * g.kv_heads, g.B), dim3(256), 0, s, g, q, ldq, cache, sink, seqlens, out, ldo, partials,
                       splits, groups);
    NC_CHECK_LAUNCH("window_few");
    if (splits > 1) {
        hipLaunchKernelGGL(window_combine_kernel, dim3(g.B * g.T * g.heads), dim3(64), 0, s, partials, splits, g.heads, g.vdim_p, g.out_scale, out, ldo);
        NC_CHECK_LAUNCH("window_combine");
    }
    return 0;
}
template <int DQ, int DV>
int launch_prefill(const NcWindowGeom& g, const bf16_t* q, int ldq, const bf16_t* cache, const float* sink, const int32_t* seqlens, bf16_t* out, int ldo,
                   hipStream_t s) {
    if ((int64_t)((g.T + 127) / 128) * g.heads * g.B >= 2 * nc_cu_count())
        hipLaunchKernelGGL((window_prefill_kernel<DQ, DV, 4, 1>), dim3((g.T + 127) / 128, g.heads, g.B), dim3(256), 0, s, g, q, ldq, cache, sink, seqlens, out, ldo);
    else
        hipLaunchKernelGGL((window_prefill_kernel<DQ, DV, 2, 2>), dim3((g.T + 63) / 64, g.heads, g.B), dim3(256), 0, s, g, q, ldq, cache, sink, seqlens, out, ldo);
    NC_CHECK_LAUNCH("window_prefill");
    return 0;
}
}  // namespace

int nc_launch_window_append(int dtype, const NcWindowGeom& g, void* proj, int ldp, const float* bias, const float* q_norm_w, const float* k_norm_w, float eps,
                            const float* rope, int rope_len, const int32_t* seqlens, void* cache, hipStream_t s) {
    NC_CHECK_ARG(g.rot_dims % 2 == 0 && g.rot_dims <= g.dim && g.dim <= g.dim_p && g.dim_p % 32 == 0 && g.vdim_p % 16 == 0, "window_append: dim=%d/%d rot=%d",
                 g.dim, g.dim_p, g.rot_dims);
    NC_CHECK_ARG(bias && q_norm_w && k_norm_w && (rope || g.rot_dims == 0) && ldp % 4 == 0, "window_append: null operand");
    NC_CHECK_ARG(g.pos_max + g.T <= rope_len && g.pos_max + g.T <= g.Tmax, "window_append: position %d past the rotary table of %d", g.pos_max + g.T, rope_len);
    NcProfScope prof(NC_CLS_ROWS, (double)g.B * g.T * (g.dim_p * (g.heads + g.kv_heads) + g.vdim_p * g.kv_heads) * (dtype ? 8 : 4), s);
    if (dtype)
        hipLaunchKernelGGL((window_append_kernel<float>), dim3(g.B * g.T), dim3(256), 0, s, g, (float*)proj, ldp, bias, q_norm_w, k_norm_w, eps, rope, rope_len,
                           seqlens, (float*)cache);
    else
        hipLaunchKernelGGL((window_append_kernel<bf16_t>), dim3(g.B * g.T), dim3(256), 0, s, g, (bf16_t*)proj, ldp, bias, q_norm_w, k_norm_w, eps, rope, rope_len,
                           seqlens, (bf16_t*)cache);
    NC_CHECK_LAUNCH("window_append");
    return 0;
}

size_t nc_window_partial_bytes(int dtype, const NcWindowGeom& g) {
    if (!mfma_ok(dtype, g) || !use_few(g)) return 0;
    const int splits = few_splits(g);
    return splits > 1 ? (size_t)g.B * g.T * g.heads * splits * (g.vdim_p + 4) * sizeof(float) : 0;
}

int nc_launch_window_attention(int dtype, const NcWindowGeom& g, const void* q, int ldq, const void* cache, const float* sink, const int32_t* seqlens, void* out,
                               int ldo, void* partials, size_t partial_bytes, hipStream_t s) {
    NC_CHECK_ARG(g.kv_heads >= 1 && g.heads % g.kv_heads == 0 && g.window >= 1 && g.keep_first >= 0, "window_attention: %d of %d heads, window %d, first %d",
                 g.kv_heads, g.heads, g.window, g.keep_first);
    NC_CHECK_ARG(g.dim_p % 32 == 0 && g.vdim_p % 16 == 0 && ldq % 8 == 0 && ldo % 4 == 0 && sink && g.pos_max + g.T <= g.Tmax, "window_attention: sizes");
    // few rows: the visible cached rows once per batch row (bytes); a prompt: (query, key) pairs (flops)
    const double es = dtype ? 4 : 2, seen = (double)g.window + g.keep_first;
    const double last = g.pos_max + g.T, keys = last < seen ? last : seen;
    const bool few = use_few(g);
    const double full = last > seen ? (last - (seen > g.pos_max ? seen : g.pos_max)) : 0, ramp_lo = g.pos_max, ramp_hi = last < seen ? last : seen;
    const double pairs = full * seen + (ramp_hi > ramp_lo ? (ramp_hi - ramp_lo) * (ramp_hi + ramp_lo + 1) * 0.5 : 0);
    NcProfScope prof(NC_CLS_WINDOW, few ? (double)g.B * keys * g.kv_heads * (g.dim_p + g.vdim_p) * es : 2.0 * g.B * g.heads * pairs * (g.dim_p + g.vdim_p), s, g.T);
    if (mfma_ok(dtype, g)) {
        const bf16_t *qq = (const bf16_t*)q, *c = (const bf16_t*)cache;
        bf16_t* o = (bf16_t*)out;
        const int splits = few ? few_splits(g) : 1;
        NC_CHECK_ARG(splits == 1 || (partials && partial_bytes >= nc_window_partial_bytes(dtype, g)), "window_attention: partial buffer too small");
#define GO(Q, V) (few ? launch_few<Q, V>(g, qq, ldq, c, sink, seqlens, o, ldo, (float*)partials, splits, s) : launch_prefill<Q, V>(g, qq, ldq, c, sink, seqlens, o, ldo, s))
#define GO_V(Q) (g.vdim_p <= 64 ? GO(Q, 64) : GO(Q, 128))
        if (g.dim_p <= 64) return GO_V(64);
        if (g.dim_p <= 128) return GO_V(128);
        return GO_V(192);
#undef GO
#undef GO_V
    }
    NC_CHECK_ARG(g.vdim_p <= 256 * SIMPLE_COLS && (g.dim_p + 256) * 4 <= 64 * 1024 - 64, "window_attention: dim=%d vdim=%d not supported", g.dim_p, g.vdim_p);
    const int bytes = (g.dim_p + 256) * 4;
    if (dtype)
        hipLaunchKernelGGL((window_simple_kernel<float>), dim3(g.B * g.T * g.heads), dim3(256), bytes, s, g, (const float*)q, ldq, (const float*)cache, sink, seqlens,
                           (float*)out, ldo);
    else
        hipLaunchKernelGGL((window_simple_kernel<bf16_t>), dim3(g.B * g.T * g.heads), dim3(256), bytes, s, g, (const bf16_t*)q, ldq, (const bf16_t*)cache, sink,
                           seqlens, (bf16_t*)out, ldo);
    NC_CHECK_LAUNCH("window_simple");
    return 0;
}
