// Retention: linear attention with one fixed decay per head.  q and k turn with the position (or not at all), k is scaled, and per head
//
//     S_t = decay S_(t-1) + k_t v_t^T   (dim x vdim, fp32),     o_t = S_t^T q_t,     y_t = o_t / rms(o_t) * silu(gate_t)
//
// or o_t itself, in fp32, where a design norms all heads together.
//
// Two forms:
//   step     token by token, the state in registers (decode, short portions, 32-bit);
//   chunked  (bf16, long portions) the sequence in chunks of C tokens: the chunks' own sums  KV_c = sum_j decay^(n-1-j) k_j v_j^T  side by
//            side, a scan over the chunks  S <- decay^n S + KV_c, and per chunk  o_i = decay^(i+1) S^T q_i + sum_(j<=i) decay^(i-j) (q_i . k_j) v_j.
// Everything that enters the recurrence is fp32.  On the matrix cores an fp32 operand goes in as two bf16 terms (hi + lo, 16 bits together):
// turned q and k, decayed k, the state, and the decayed scores; products of two lo terms are left out.
//
// State layout fp32 [batch][heads][dim_p][vdim_p]; a row at position 0 starts from zero and does not read its state.
#include "nc_stack.h"

typedef __bf16 v8bf __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
typedef short v4s __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) v4s* lds_v4s_t;
typedef __attribute__((address_space(3))) uint8_t* lds_u8_t;

namespace {
__device__ __forceinline__ v8bf as_v8bf(uint4 v) { return __builtin_bit_cast(v8bf, v); }
__device__ __forceinline__ void split8(const float* v, v8bf& hi, v8bf& lo) {
#pragma unroll
    for (int j = 0; j < 8; j++) {
        hi[j] = (__bf16)v[j];
        lo[j] = (__bf16)(v[j] - (float)hi[j]);
    }
}
__device__ __forceinline__ v8bf tr_read8(lds_u8_t p, int second) {
    const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)p);
    const v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s_t)(p + second));
    return __builtin_bit_cast(v8bf, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}
// dimension d of a turned vector: (u, v) = (x_i, x_(i+half)) -> (u cos - v sin, v cos + u sin)
template <typename T>
__device__ __forceinline__ float turned(const T* x, int d, int half, const float2* turn) {
    const float a = ld_f32(x + d);
    if (d < half) return a * turn[d].x - ld_f32(x + d + half) * turn[d].y;
    if (d < 2 * half) return a * turn[d - half].x + ld_f32(x + d - half) * turn[d - half].y;
    return a;
}
// eight consecutive dimensions from d0 (a multiple of 8) of a turned bf16 vector, times `scale`
__device__ __forceinline__ void turned8(const bf16_t* x, int d0, int half, const float2* turn, float scale, float (&out)[8]) {
    if ((half & 7) == 0) {                 // uniform: the partners are eight consecutive dimensions as well
        const v4f a0 = ld4_f32(x + d0), a1 = ld4_f32(x + d0 + 4);
        float a[8] = {a0[0], a0[1], a0[2], a0[3], a1[0], a1[1], a1[2], a1[3]};
        if (d0 < 2 * half) {
            const bool first = d0 < half;
            const int dp = first ? d0 + half : d0 - half;
            const float2* w = turn + (first ? d0 : dp);
            const float sign = first ? -1.f : 1.f;
            const v4f p0 = ld4_f32(x + dp), p1 = ld4_f32(x + dp + 4);
            const float p[8] = {p0[0], p0[1], p0[2], p0[3], p1[0], p1[1], p1[2], p1[3]};
#pragma unroll
            for (int j = 0; j < 8; j++) a[j] = a[j] * w[j].x + sign * (p[j] * w[j].y);
        }
#pragma unroll
        for (int j = 0; j < 8; j++) out[j] = a[j] * scale;
    } else {
#pragma unroll
        for (int j = 0; j < 8; j++) out[j] = turned(x, d0 + j, half, turn) * scale;
    }
}

// ------------------------------------------------------------------------------------------------ step
// One workgroup per (head, batch row).  Thread (kg, vg) holds S[kg + KG i][4 vg .. + 3]; a token costs one pass over the registers and a
// sum over the kg through LDS.
template <typename T, int DK, int DV, int NTHR>
__global__ __launch_bounds__(NTHR) void retention_step_kernel(NcRetentionGeom g, const T* __restrict__ proj, int ldp, const float* __restrict__ decay,
                                                              const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                              const float* __restrict__ state_in, float* __restrict__ state_out, float eps,
                                                              T* __restrict__ out, int ldo) {
    constexpr int VG = DV / 4, KG = NTHR / VG, KI = DK / KG;
    static_assert(DK % KG == 0 && VG <= 64, "sizes");
    __shared__ float qs[DK], ks[DK];
    __shared__ v4f part[KG][VG];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, vg = tid % VG, kg = tid / VG;
    const int pos0 = seqlens[b], half = g.rot_dims / 2;
    const int64_t so = ((int64_t)b * g.heads + h) * DK * DV + kg * DV + 4 * vg;
    v4f S[KI];
    if (pos0 > 0) {
#pragma unroll
        for (int i = 0; i < KI; i++) S[i] = __builtin_nontemporal_load((const v4f*)(state_in + so + (int64_t)i * KG * DV));
    } else {
#pragma unroll
        for (int i = 0; i < KI; i++) S[i] = v4f{0.f, 0.f, 0.f, 0.f};
    }
    const float dec = decay[2 * h];
    for (int t = 0; t < g.T; t++) {
        const int64_t m = (int64_t)b * g.T + t;
        const T* row = proj + m * ldp;
        const T *q = row + h * DK, *k = row + (g.heads + h) * DK, *v = row + 2 * g.heads * DK + h * DV, *gate = v + g.heads * DV;
        const float2* turn = (const float2*)rope + (int64_t)min(pos0 + t, rope_len - 1) * half;
        for (int d = tid; d < DK; d += NTHR) {
            qs[d] = turned(q, d, half, turn);
            ks[d] = turned(k, d, half, turn) * g.k_scale;
        }
        const v4f vv = ld4_f32(v + 4 * vg);
        __syncthreads();
        v4f o = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KI; i++) {
            S[i] = S[i] * dec + vv * ks[kg + KG * i];
            o += S[i] * qs[kg + KG * i];
        }
        part[kg][vg] = o;
        __syncthreads();
        if (tid < 64) {
            v4f y = v4f{0.f, 0.f, 0.f, 0.f};
            if (tid < VG)
                for (int i = 0; i < KG; i++) y += part[i][tid];
            const float ss = wave_sum((y[0] * y[0] + y[1] * y[1]) + (y[2] * y[2] + y[3] * y[3]));
            const float inv = 1.0f / sqrtf(ss / (float)g.vdim + eps);
            const int c = h * g.vdim_p + 4 * tid;
            if (g.raw) {
                if (tid < VG) *(v4f*)(g.raw + m * g.heads * g.vdim_p + c) = y;
            } else if (tid < VG) {
                const v4f z = ld4_f32(gate + 4 * tid);
                v4f r;
#pragma unroll
                for (int j = 0; j < 4; j++) r[j] = y[j] * inv * (z[j] * sigmoid_f32(z[j]));
                st4_f32(out + m * ldo + c, r);
            }
        }
        // (the next token's qs / ks are written before the next barrier, by threads that are past the loop above; `part` after it)
    }
#pragma unroll
    for (int i = 0; i < KI; i++) __builtin_nontemporal_store(S[i], (v4f*)(state_out + so + (int64_t)i * KG * DV));
}

// Any sizes: the state stays in memory (state_out), a thread owns value columns.
template <typename T>
__global__ __launch_bounds__(256) void retention_plain_kernel(NcRetentionGeom g, const T* __restrict__ proj, int ldp, const float* __restrict__ decay,
                                                              const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                              const float* __restrict__ state_in, float* __restrict__ state_out, float eps,
                                                              T* __restrict__ out, int ldo) {
    extern __shared__ float sh[];          // q | k | o
    __shared__ float red[4];
    float *qs = sh, *ks = sh + g.dim_p, *os = sh + 2 * g.dim_p;
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, half = g.rot_dims / 2, pos0 = seqlens[b];
    const int64_t so = ((int64_t)b * g.heads + h) * g.dim_p * g.vdim_p;
    const float dec = decay[2 * h];
    for (int t = 0; t < g.T; t++) {
        const int64_t m = (int64_t)b * g.T + t;
        const T* row = proj + m * ldp;
        const T *q = row + h * g.dim_p, *k = row + (g.heads + h) * g.dim_p, *v = row + 2 * g.heads * g.dim_p + h * g.vdim_p, *gate = v + g.heads * g.vdim_p;
        const float2* turn = (const float2*)rope + (int64_t)min(pos0 + t, rope_len - 1) * half;
        __syncthreads();
        for (int d = tid; d < g.dim_p; d += 256) {
            qs[d] = turned(q, d, half, turn);
            ks[d] = turned(k, d, half, turn) * g.k_scale;
        }
        __syncthreads();
        float ss = 0.f;
        for (int c = tid; c < g.vdim_p; c += 256) {
            const float vv = ld_f32(v + c);
            float o = 0.f;
            for (int d = 0; d < g.dim_p; d++) {
                const int64_t at = so + (int64_t)d * g.vdim_p + c;
                const float s = t > 0 ? state_out[at] : pos0 > 0 ? state_in[at] : 0.f;
                const float n = s * dec + vv * ks[d];
                state_out[at] = n;
                o += n * qs[d];
            }
            os[c] = o;
            ss += o * o;
        }
        const float inv = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)g.vdim + eps);
        for (int c = tid; c < g.vdim_p; c += 256) {
            if (g.raw) {
                g.raw[(m * g.heads + h) * g.vdim_p + c] = os[c];
                continue;
            }
            const float z = ld_f32(gate + c);
            st_f32(out + m * ldo + h * g.vdim_p + c, os[c] * inv * (z * sigmoid_f32(z)));
        }
    }
}

// ------------------------------------------------------------------------------------------------ chunked
// KV_c^T [vdim][dim] of one chunk and head.  Waves take 32 x 32 tiles in turn; both operands through the transposing LDS read.
template <int DK, int DV, int C>
__global__ __launch_bounds__(256) void retention_chunk_kv_kernel(NcRetentionGeom g, const bf16_t* __restrict__ proj, int ldp, const float* __restrict__ decay,
                                                                 const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                                 float* __restrict__ kv, int chunks) {
    constexpr int KP = DK * 2 + 64, VP = DV * 2 + 64, TILES = (DK / 32) * (DV / 32), PER = (TILES + 3) / 4;
    __shared__ __align__(16) uint8_t lds[C * (2 * KP + VP)];
    uint8_t *const lk_hi = lds, *const lk_lo = lds + C * KP, *const lv = lds + 2 * C * KP;
    const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int half = g.rot_dims / 2, pos0 = seqlens[b], n = min(C, g.T - chunk * C);
    const float l2 = decay[2 * h + 1];
    for (int u = tid; u < C * DK / 8; u += 256) {
        const int j = u / (DK / 8), d0 = 8 * (u % (DK / 8));
        v8bf hi, lo;
        float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (j < n) {
            const int t = chunk * C + j;
            turned8(proj + ((int64_t)b * g.T + t) * ldp + (g.heads + h) * DK, d0, half, (const float2*)rope + (int64_t)min(pos0 + t, rope_len - 1) * half,
                    g.k_scale * exp2f((float)(n - 1 - j) * l2), x);
        }
        split8(x, hi, lo);
        *(v8bf*)(lk_hi + j * KP + d0 * 2) = hi;
        *(v8bf*)(lk_lo + j * KP + d0 * 2) = lo;
    }
    for (int u = tid; u < C * DV / 8; u += 256) {
        const int j = u / (DV / 8), d0 = 8 * (u % (DV / 8));
        uint4 v = make_uint4(0, 0, 0, 0);
        if (j < n) v = *(const uint4*)(proj + ((int64_t)b * g.T + chunk * C + j) * ldp + 2 * g.heads * DK + h * DV + d0);
        *(uint4*)(lv + j * VP + d0 * 2) = v;
    }
    __syncthreads();
    // this lane's place inside a 16-token, 32-column block of the transposing read (first four tokens; the second four lie 8 rows on)
    const int trow = 4 * (lane >> 5) + ((lane & 15) >> 2), tcol = 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
    const lds_u8_t l3 = (lds_u8_t)lds;
    float* dst = kv + (((int64_t)b * chunks + chunk) * g.heads + h) * DK * DV;
#pragma unroll
    for (int p = 0; p < PER; p++) {
        const int tile = wave + 4 * p;
        if (tile >= TILES) break;
        const int tv = tile / (DK / 32), tk = tile % (DK / 32);
        v16f acc;
#pragma unroll
        for (int r = 0; r < 16; r++) acc[r] = 0.f;
#pragma unroll
        for (int c = 0; c < C / 16; c++) {
            const v8bf vf = tr_read8(l3 + 2 * C * KP + (16 * c + trow) * VP + (32 * tv + tcol) * 2, 8 * VP);
            const v8bf kh = tr_read8(l3 + (16 * c + trow) * KP + (32 * tk + tcol) * 2, 8 * KP);
            const v8bf kl = tr_read8(l3 + C * KP + (16 * c + trow) * KP + (32 * tk + tcol) * 2, 8 * KP);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, kh, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, kl, acc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 16; r++)
            dst[(int64_t)(32 * tv + 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3)) * DK + 32 * tk + (lane & 31)] = acc[r];
    }
}

// The state in front of every chunk, as two bf16 terms (hi, then lo DK * DV elements on), and the state behind the last one.  The terms are
// laid out as the operand of S^T q reads them: 32 value rows x 16 dims are 64 lanes x 8 elements, lane = row % 32 + 32 (dim % 16 / 8).
// One thread per four elements of S^T [vdim][dim].
__global__ __launch_bounds__(256) void retention_scan_kernel(NcRetentionGeom g, const float* __restrict__ decay, const int32_t* __restrict__ seqlens,
                                                             const float* __restrict__ kv, bf16_t* __restrict__ prefix,
                                                             const float* __restrict__ state_in, float* __restrict__ state_out, int chunks, int C) {
    const int h = blockIdx.y, b = blockIdx.z, DK = g.dim_p, DV = g.vdim_p;
    const int e = 4 * ((int)blockIdx.x * 256 + (int)threadIdx.x);
    if (e >= DK * DV) return;
    const int v = e / DK, k = e % DK;
    const int64_t so = ((int64_t)b * g.heads + h) * DK * DV;
    v4f S = v4f{0.f, 0.f, 0.f, 0.f};
    if (seqlens[b] > 0)
#pragma unroll
        for (int j = 0; j < 4; j++) S[j] = state_in[so + (int64_t)(k + j) * DV + v];
    const float l2 = decay[2 * h + 1];
    const float full = exp2f((float)C * l2), tail = exp2f((float)(g.T - (chunks - 1) * C) * l2);
    const int64_t step = (int64_t)g.heads * DK * DV;
    const float* src = kv + (((int64_t)b * chunks) * g.heads + h) * DK * DV + e;
    const int place = ((v / 32 * (DK / 16) + k / 16) * 64 + v % 32 + 32 * (k % 16 / 8)) * 8 + k % 8;
    bf16_t* dst = prefix + 2 * ((((int64_t)b * chunks) * g.heads + h) * DK * DV) + place;
#pragma unroll 4
    for (int c = 0; c < chunks; c++) {
        const v4f add = *(const v4f*)(src + c * step);
        v4f lo;
#pragma unroll
        for (int j = 0; j < 4; j++) lo[j] = S[j] - rbf(S[j]);
        st4_f32(dst + 2 * c * step, S);
        st4_f32(dst + 2 * c * step + DK * DV, lo);
        S = S * (c + 1 < chunks ? full : tail) + add;
    }
#pragma unroll
    for (int j = 0; j < 4; j++) state_out[so + (int64_t)(k + j) * DV + v] = S[j];
}

// The outputs of one chunk and head.  Four waves: C / 32 blocks of 32 queries x the value columns dealt to 4 / (C / 32) waves, each of which
// computes the scores of its queries for itself.  Transposed like the attention kernels (a lane owns one query): S^T = K Q^T, O^T = V^T P^T.
template <int DK, int DV, int C>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) void retention_chunk_out_kernel(NcRetentionGeom g, const bf16_t* __restrict__ proj, int ldp, const float* __restrict__ decay,
                                                                  const float* __restrict__ rope, int rope_len, const int32_t* __restrict__ seqlens,
                                                                  const bf16_t* __restrict__ prefix, int chunks, float eps, bf16_t* __restrict__ out, int ldo) {
    constexpr int QB = C / 32, VS = 4 / QB, NT = DV / 32 / VS, KP = DK * 2 + 16, VP = DV * 2 + 64;
    static_assert(NT >= 1, "value columns per wave");
    __shared__ __align__(16) uint8_t lds[C * (2 * KP + VP)];
    __shared__ float red[VS][C];
    uint8_t *const lk_hi = lds, *const lk_lo = lds + C * KP, *const lv = lds + 2 * C * KP;
    const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), qb = wave % QB, vs = wave / QB;
    const int col = lane & 31, hl = lane >> 5;
    const int half = g.rot_dims / 2, pos0 = seqlens[b], t0 = chunk * C, n = min(C, g.T - t0);
    const float l2 = decay[2 * h + 1];
    const bf16_t* base = proj + ((int64_t)b * g.T + t0) * ldp;
    const float2* turns = (const float2*)rope;

    for (int u = tid; u < C * DK / 8; u += 256) {
        const int j = u / (DK / 8), d0 = 8 * (u % (DK / 8)), jj = min(j, n - 1);
        float x[8];
        turned8(base + (int64_t)jj * ldp + (g.heads + h) * DK, d0, half, turns + (int64_t)min(pos0 + t0 + jj, rope_len - 1) * half, g.k_scale, x);
        v8bf hi, lo;
        split8(x, hi, lo);
        *(v8bf*)(lk_hi + j * KP + d0 * 2) = hi;
        *(v8bf*)(lk_lo + j * KP + d0 * 2) = lo;
    }
    for (int u = tid; u < C * DV / 8; u += 256) {
        const int j = u / (DV / 8), d0 = 8 * (u % (DV / 8)), jj = min(j, n - 1);
        *(uint4*)(lv + j * VP + d0 * 2) = *(const uint4*)(base + (int64_t)jj * ldp + 2 * g.heads * DK + h * DV + d0);
    }
    // this lane's query, turned
    const int i = 32 * qb + col, iq = min(i, n - 1);
    v8bf qh[DK / 16], ql[DK / 16];
#pragma unroll
    for (int c = 0; c < DK / 16; c++) {
        float x[8];
        turned8(base + (int64_t)iq * ldp + h * DK, 16 * c + 8 * hl, half, turns + (int64_t)min(pos0 + t0 + iq, rope_len - 1) * half, 1.0f, x);
        split8(x, qh[c], ql[c]);
    }
    v16f o[NT];
#pragma unroll
    for (int d = 0; d < NT; d++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[d][r] = 0.f;
    if (chunk > 0 || pos0 > 0) {            // what came before the chunk
        const bf16_t* st = prefix + 2 * ((((int64_t)b * chunks + chunk) * g.heads + h) * DK * DV);
#pragma unroll
        for (int d = 0; d < NT; d++) {
            const bf16_t* srow = st + ((int64_t)(vs * NT + d) * (DK / 16) * 64 + lane) * 8;
#pragma unroll
            for (int c = 0; c < DK / 16; c++) {
                const v8bf sh = as_v8bf(*(const uint4*)(srow + 512 * c)), sl = as_v8bf(*(const uint4*)(srow + DK * DV + 512 * c));
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sh, qh[c], o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sh, ql[c], o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sl, qh[c], o[d], 0, 0, 0);
            }
        }
        const float w = exp2f((float)(i + 1) * l2);
#pragma unroll
        for (int d = 0; d < NT; d++)
#pragma unroll
            for (int r = 0; r < 16; r++) o[d][r] *= w;
    }
    __syncthreads();
    const lds_u8_t l3v = (lds_u8_t)lds + 2 * C * KP + (4 * hl + ((lane & 15) >> 2)) * VP + (16 * ((lane >> 4) & 1) + 4 * (lane & 3)) * 2;
#pragma unroll 1
    for (int sb = 0; sb <= qb; sb++) {
        v16f s;
#pragma unroll
        for (int r = 0; r < 16; r++) s[r] = 0.f;
        const uint8_t *kh = lk_hi + (32 * sb + col) * KP + 16 * hl, *kl = lk_lo + (32 * sb + col) * KP + 16 * hl;
#pragma unroll
        for (int c = 0; c < DK / 16; c++) {
            const v8bf fh = as_v8bf(*(const uint4*)(kh + 32 * c)), fl = as_v8bf(*(const uint4*)(kl + 32 * c));
            s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fh, qh[c], s, 0, 0, 0);
            s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fh, ql[c], s, 0, 0, 0);
            s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fl, qh[c], s, 0, 0, 0);
        }
        v8bf ph[2], pl[2];
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int j = 32 * sb + 8 * (r >> 2) + 4 * hl + (r & 3);
            const float w = j <= i ? s[r] * __builtin_amdgcn_exp2f((float)(i - j) * l2) : 0.f;
            ph[r >> 3][r & 7] = (__bf16)w;
            pl[r >> 3][r & 7] = (__bf16)(w - (float)ph[r >> 3][r & 7]);
        }
#pragma unroll
        for (int c2 = 0; c2 < 2; c2++)
#pragma unroll
            for (int d = 0; d < NT; d++) {
                const v8bf vf = tr_read8(l3v + (32 * sb + 16 * c2) * VP + 64 * (vs * NT + d), 8 * VP);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, ph[c2], o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pl[c2], o[d], 0, 0, 0);
            }
    }
    if (g.raw) {                               // (uniform)
        if (i >= n) return;
        float* row = g.raw + (((int64_t)b * g.T + t0 + i) * g.heads + h) * DV;
#pragma unroll
        for (int d = 0; d < NT; d++)
#pragma unroll
            for (int g4 = 0; g4 < 4; g4++)
                *(v4f*)(row + 32 * (vs * NT + d) + 8 * g4 + 4 * hl) = v4f{o[d][4 * g4], o[d][4 * g4 + 1], o[d][4 * g4 + 2], o[d][4 * g4 + 3]};
        return;
    }
    float ss = 0.f;
#pragma unroll
    for (int d = 0; d < NT; d++)
#pragma unroll
        for (int r = 0; r < 16; r++) ss = fmaf(o[d][r], o[d][r], ss);
    ss += __shfl_xor(ss, 32);
    if (hl == 0) red[vs][i] = ss;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < VS; w++) tot += red[w][i];
    if (i >= n) return;
    const float inv = 1.0f / sqrtf(tot / (float)g.vdim + eps);
    const bf16_t* gate = base + (int64_t)i * ldp + 2 * g.heads * DK + (g.heads + h) * DV;
    bf16_t* orow = out + ((int64_t)b * g.T + t0 + i) * ldo + h * DV;
#pragma unroll
    for (int d = 0; d < NT; d++)
#pragma unroll
        for (int g4 = 0; g4 < 4; g4++) {
            const int c = 32 * (vs * NT + d) + 8 * g4 + 4 * hl;
            const v4f z = ld4_f32(gate + c);
            v4f r;
#pragma unroll
            for (int j = 0; j < 4; j++) r[j] = o[d][4 * g4 + j] * inv * (z[j] * sigmoid_f32(z[j]));
            st4_f32(orow + c, r);
        }
}

constexpr int CHUNK_MIN_TOKENS = 32;
int chunk_size(int dtype, const NcRetentionGeom& g) {
    if (dtype != 0 || g.T < CHUNK_MIN_TOKENS) return 0;
    if ((g.dim_p == 64 || g.dim_p == 128) && (g.vdim_p == 64 || g.vdim_p == 128 || g.vdim_p == 256)) return 64;
    if (g.dim_p == 256 && (g.vdim_p == 128 || g.vdim_p == 256)) return 32;
    return 0;
}
template <int DK, int DV, int C>
int launch_chunked(const NcRetentionGeom& g, const bf16_t* proj, int ldp, const float* decay, const float* rope, int rope_len, const int32_t* seqlens,
                   const float* state_in, float* state_out, float eps, bf16_t* out, int ldo, void* workspace, hipStream_t s) {
    const int chunks = (g.T + C - 1) / C;
    float* kv = (float*)workspace;
    bf16_t* prefix = (bf16_t*)(kv + (int64_t)g.B * chunks * g.heads * DK * DV);
    hipLaunchKernelGGL((retention_chunk_kv_kernel<DK, DV, C>), dim3(chunks, g.heads, g.B), dim3(256), 0, s, g, proj, ldp, decay, rope, rope_len, seqlens, kv,
                       chunks);
    hipLaunchKernelGGL(retention_scan_kernel, dim3((DK * DV + 1023) / 1024, g.heads, g.B), dim3(256), 0, s, g, decay, seqlens, kv, prefix, state_in, state_out,
                       chunks, C);
    hipLaunchKernelGGL((retention_chunk_out_kernel<DK, DV, C>), dim3(chunks, g.heads, g.B), dim3(256), 0, s, g, proj, ldp, decay, rope, rope_len, seqlens,
                       prefix, chunks, eps, out, ldo);
    NC_CHECK_LAUNCH("retention_chunked");
    return 0;
}
template <typename T>
int launch_step(const NcRetentionGeom& g, const T* proj, int ldp, const float* decay, const float* rope, int rope_len, const int32_t* seqlens,
                const float* state_in, float* state_out, float eps, T* out, int ldo, hipStream_t s) {
#define STEP(K, V, N)                                                                                                                            \
    if (g.dim_p == K && g.vdim_p == V) {                                                                                                         \
        hipLaunchKernelGGL((retention_step_kernel<T, K, V, N>), dim3(g.heads, g.B), dim3(N), 0, s, g, proj, ldp, decay, rope, rope_len, seqlens, \
                           state_in, state_out, eps, out, ldo);                                                                                  \
        NC_CHECK_LAUNCH("retention_step");                                                                                                       \
        return 0;                                                                                                                                \
    }
    STEP(64, 64, 256) STEP(64, 128, 256) STEP(64, 256, 512) STEP(128, 64, 256) STEP(128, 128, 512) STEP(128, 256, 1024) STEP(256, 128, 1024)
    STEP(256, 256, 1024)
#undef STEP
    hipLaunchKernelGGL((retention_plain_kernel<T>), dim3(g.heads, g.B), dim3(256), (2 * g.dim_p + g.vdim_p) * 4, s, g, proj, ldp, decay, rope, rope_len,
                       seqlens, state_in, state_out, eps, out, ldo);
    NC_CHECK_LAUNCH("retention_plain");
    return 0;
}
}  // namespace

size_t nc_retention_workspace_bytes(int dtype, const NcRetentionGeom& g) {
    const int C = chunk_size(dtype, g);
    return C ? (size_t)g.B * ((g.T + C - 1) / C) * g.heads * g.dim_p * g.vdim_p * 8 : 0;
}

int nc_launch_retention(int dtype, const NcRetentionGeom& g, const void* proj, int ldp, const float* decay, const float* rope, int rope_len,
                        const int32_t* seqlens, const float* state_in, float* state_out, float eps, void* out, int ldo, void* workspace,
                        hipStream_t s) {
    NC_CHECK_ARG(g.rot_dims % 2 == 0 && g.rot_dims <= g.dim && g.dim <= g.dim_p && g.vdim <= g.vdim_p && g.dim_p % 8 == 0 && g.vdim_p % 8 == 0,
                 "retention: dim=%d/%d vdim=%d/%d rot=%d", g.dim, g.dim_p, g.vdim, g.vdim_p, g.rot_dims);
    NC_CHECK_ARG(state_in != state_out, "retention: the state is not updated in place");
    NC_CHECK_ARG((2 * g.dim_p + g.vdim_p) * 4 <= 64 * 1024, "retention: dim=%d vdim=%d not supported", g.dim_p, g.vdim_p);
    const int C = chunk_size(dtype, g);
    if (!C) {
        // the state once in and once out (bytes); per token the projections
        NcProfScope prof(NC_CLS_RETENTION, (double)g.B * g.heads * (8.0 * g.dim_p * g.vdim_p + (double)g.T * (2 * g.dim_p + 3 * g.vdim_p) * (dtype ? 4 : 2)), s, g.T);
        return dtype ? launch_step<float>(g, (const float*)proj, ldp, decay, rope, rope_len, seqlens, state_in, state_out, eps, (float*)out, ldo, s)
                     : launch_step<bf16_t>(g, (const bf16_t*)proj, ldp, decay, rope, rope_len, seqlens, state_in, state_out, eps, (bf16_t*)out, ldo, s);
    }
    // bytes: the projections in, the outputs, and four passes over the chunks' states (written, scanned in and out, read)
    NcProfScope prof(NC_CLS_RETENTION, (double)g.B * g.heads * (g.T * (2.0 * g.dim_p + 3.0 * g.vdim_p) * 2 + 16.0 * ((g.T + C - 1) / C) * g.dim_p * g.vdim_p), s,
                     g.T);
    const bf16_t* p = (const bf16_t*)proj;
    bf16_t* o = (bf16_t*)out;
#define CHUNKED(K, V, CC) \
    if (g.dim_p == K && g.vdim_p == V) return launch_chunked<K, V, CC>(g, p, ldp, decay, rope, rope_len, seqlens, state_in, state_out, eps, o, ldo, workspace, s);
    CHUNKED(64, 64, 64) CHUNKED(64, 128, 64) CHUNKED(64, 256, 64) CHUNKED(128, 64, 64) CHUNKED(128, 128, 64) CHUNKED(128, 256, 64)
    CHUNKED(256, 128, 32) CHUNKED(256, 256, 32)
#undef CHUNKED
    NC_FAIL(-1, "retention: no chunked kernel for %d x %d", g.dim_p, g.vdim_p);
}
