// Selective scan: a causal convolution per channel, then per channel c and state n a linear recurrence whose step comes from the token,
//
//     S[c,n] <- exp(dt_c A[c,n]) S[c,n] + dt_c u_c B_n,     y_c = (sum_n S[c,n] C_n + D_c u_c) silu(z_c)
//
// with dt (softplus done by the linear that makes it), B and C per token.  State fp32, kept [state_p + taps - 1][inner_p] per sequence: the
// recurrent state, then the last inputs of the convolution.  A row at position 0 starts from zero and does not read its state.
//
// A channel's states are dealt to LG lanes, SP to each, in registers: lane = part * (64 / LG) + channel, so that neighbours read
// neighbouring channels.  Tokens go TB at a time: their B and C through LDS (every channel reads the same ones), a lane's own dt, u and z
// into registers ahead of their use.
//   step        one token per row (decode): from the shares of the product that gives dt, B and C to the result in one launch
//   one pass    short portions: the tokens one after the other
//   chunked     long portions: every chunk's own sums from a zero state side by side, a scan over the chunks
//               S <- exp(A sum dt) S + own sums, then every chunk again from its true start, with outputs
// A is kept times log2(e), so that a decay is one exp2.
#include "nc_stack.h"

namespace {
constexpr int TB = 8;
enum { SCAN_WHOLE = 0, SCAN_SUMS = 1, SCAN_OUT = 2 };

// Four channels and CONV_TOKENS tokens per thread, the inputs sliding through registers (up to MAX_TAPS of them; more are read again).
constexpr int CONV_TOKENS = 8, MAX_TAPS = 4;
template <typename T>
__global__ __launch_bounds__(256) void scan_conv_kernel(NcScanGeom g, const T* __restrict__ x, int ldx, const float* __restrict__ w, const float* __restrict__ bias,
                                                        const int32_t* __restrict__ seqlens, const float* __restrict__ state_in, float* __restrict__ state_out,
                                                        T* __restrict__ u) {
    const int c = 4 * ((int)blockIdx.x * 256 + (int)threadIdx.x), t0 = (int)blockIdx.y * CONV_TOKENS, b = blockIdx.z;
    if (c >= g.inner_p) return;
    const int old = g.taps - 1;
    const bool fresh = seqlens[b] == 0;
    const int64_t so = ((int64_t)b * (g.state_p + old) + g.state_p) * g.inner_p + c;
    // input of token tt of this portion; earlier ones come out of the state, oldest first
    auto input = [&](int tt) -> v4f {
        if (tt >= 0) return ld4_f32(x + ((int64_t)b * g.T + min(tt, g.T - 1)) * ldx + c);
        if (fresh) return v4f{0.f, 0.f, 0.f, 0.f};
        return *(const v4f*)(state_in + so + (int64_t)(old + tt) * g.inner_p);
    };
    const v4f bv = *(const v4f*)(bias + c);
    auto store = [&](int t, v4f y) {
        st4_f32(u + ((int64_t)b * g.T + t) * g.inner_p + c, v4f{silu_f32(y[0]), silu_f32(y[1]), silu_f32(y[2]), silu_f32(y[3])});
    };
    if (g.taps == MAX_TAPS) {                               // (uniform)
        v4f wv[MAX_TAPS], in[CONV_TOKENS + MAX_TAPS - 1];
#pragma unroll
        for (int i = 0; i < MAX_TAPS; i++) wv[i] = *(const v4f*)(w + (int64_t)i * g.inner_p + c);
#pragma unroll
        for (int i = 0; i < CONV_TOKENS + MAX_TAPS - 1; i++)
            if (i < MAX_TAPS || t0 + i - old < g.T) in[i] = input(t0 + i - old);
            else in[i] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < CONV_TOKENS; j++) {
            if (t0 + j >= g.T) break;
            v4f y = bv;
#pragma unroll
            for (int i = 0; i < MAX_TAPS; i++) y += wv[i] * in[j + i];
            store(t0 + j, y);
        }
    } else {
        for (int t = t0; t < min(t0 + CONV_TOKENS, g.T); t++) {
            v4f y = bv;
            for (int i = 0; i < g.taps; i++) y += *(const v4f*)(w + (int64_t)i * g.inner_p + c) * input(t - old + i);
            store(t, y);
        }
    }
    if (t0 + CONV_TOKENS >= g.T)
        for (int j = 0; j < old; j++) *(v4f*)(state_out + so + (int64_t)j * g.inner_p) = input(g.T - old + j);
}

// One thread per four columns of one row.
template <typename T>
__global__ __launch_bounds__(256) void scan_join_kernel(const float* __restrict__ parts, int splits, int64_t M, int rank_p, int bc_cols, T* __restrict__ dtr,
                                                        float* __restrict__ bc) {
    const int N = rank_p + 2 * bc_cols;
    const int64_t e = 4 * ((int64_t)blockIdx.x * 256 + threadIdx.x);
    if (e >= M * N) return;
    v4f p[8], sum = v4f{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < splits; s0 += 8) {
#pragma unroll
        for (int s = 0; s < 8; s++) p[s] = *(const v4f*)(parts + min(s0 + s, splits - 1) * M * N + e);
#pragma unroll
        for (int s = 0; s < 8; s++)
            if (s0 + s < splits) sum += p[s];
    }
    const int64_t m = e / N;
    const int n = (int)(e % N);
    if (n < rank_p) st4_f32(dtr + m * rank_p + n, sum);
    else *(v4f*)(bc + m * 2 * bc_cols + n - rank_p) = sum;
}

// One token per row.  A workgroup of four waves takes 64 channels (one per lane) and RB rows: the waves share the sum over the step's rank,
// then the states (SPW at most each); partial sums meet in LDS.
template <typename T, int RB, int SPW>
__global__ __launch_bounds__(256) void scan_step_kernel(NcScanGeom g, NcScanStep p) {
    extern __shared__ __align__(16) float lds[];             // the rows' [step before W_dt | B | C]
    __shared__ float red[4][RB][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c = (int)blockIdx.x * 64 + lane, b0 = (int)blockIdx.y * RB, rows = min(RB, g.B - b0);
    const int bc_cols = nc_scan_bc_cols(g.state_p), N = g.dt_rank_p + 2 * bc_cols, per = g.state_p / 4, n0 = wave * per;
    const int64_t plane = (int64_t)(g.state_p + g.taps - 1) * g.inner_p;
    // Loads come back in the order they are asked for: first what the first barrier waits for (the shares), then 16 weights of this wave's
    // part of the sum over the step's rank, then the state, which nobody needs before the second barrier.
    auto shares = [&](int i, int s0, v4f (&v)[8]) {
        const float* src = p.parts + (int64_t)b0 * N + i;
#pragma unroll
        for (int s = 0; s < 8; s++) v[s] = *(const v4f*)(src + (int64_t)min(s0 + s, p.splits - 1) * g.B * N);
    };
    v4f first[8];
    const int i0 = min(4 * tid, rows * N - 4);
    shares(i0, 0, first);
    const int share = g.dt_rank_p / 4, k0 = wave * share;    // a multiple of 16
    const T* wp = (const T*)p.w_dt_t + (int64_t)k0 * g.inner_p + c;
    T wv[16];
#pragma unroll
    for (int j = 0; j < 16; j++) wv[j] = wp[(int64_t)j * g.inner_p];
    float S[RB][SPW], a[SPW], uv[RB], zv[RB];
    bool fresh[RB];
#pragma unroll
    for (int r = 0; r < RB; r++) {
        const int b = b0 + min(r, rows - 1);
        fresh[r] = p.seqlens[b] == 0;
        uv[r] = ld_f32((const T*)p.u + (int64_t)b * g.inner_p + c);
        zv[r] = ld_f32((const T*)p.z + (int64_t)b * p.ldz + c);
#pragma unroll
        for (int i = 0; i < SPW; i++) S[r][i] = p.state_in[b * plane + (int64_t)(n0 + min(i, per - 1)) * g.inner_p + c];
    }
#pragma unroll
    for (int i = 0; i < SPW; i++) a[i] = p.a_log2[(int64_t)(n0 + min(i, per - 1)) * g.inner_p + c];
    const float bias = p.dt_b[c], d = p.skip[c];
    for (int i = 4 * tid; i < rows * N; i += 1024) {
        v4f sum = v4f{0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < p.splits; s0 += 8) {
            if (s0 > 0 || i >= 1024) shares(i, s0, first);
#pragma unroll
            for (int s = 0; s < 8; s++)
                if (s0 + s < p.splits) sum += first[s];
        }
        *(v4f*)(lds + i) = sum;
    }
    __syncthreads();
    float dt[RB];
#pragma unroll
    for (int r = 0; r < RB; r++) dt[r] = 0.f;
#pragma unroll 1
    for (int k = 0; k < share; k += 16) {
        float w[16];
#pragma unroll
        for (int j = 0; j < 16; j++) w[j] = ld_f32(&wv[j]);
        if (k + 16 < share)
#pragma unroll
            for (int j = 0; j < 16; j++) wv[j] = wp[(int64_t)(k + 16 + j) * g.inner_p];
#pragma unroll
        for (int j = 0; j < 16; j += 4)
#pragma unroll
            for (int r = 0; r < RB; r++) {
                const v4f x = *(const v4f*)(lds + min(r, rows - 1) * N + k0 + k + j);
                dt[r] = fmaf(w[j + 3], x[3], fmaf(w[j + 2], x[2], fmaf(w[j + 1], x[1], fmaf(w[j], x[0], dt[r]))));
            }
    }
#pragma unroll
    for (int r = 0; r < RB; r++) red[wave][r][lane] = dt[r];
    __syncthreads();
    float y[RB];
#pragma unroll
    for (int r = 0; r < RB; r++) {
        dt[r] = softplus_f32((red[0][r][lane] + red[1][r][lane]) + (red[2][r][lane] + red[3][r][lane]) + bias);
        const float* bj = lds + min(r, rows - 1) * N + g.dt_rank_p + n0;
        const float du = dt[r] * uv[r];
        y[r] = 0.f;
#pragma unroll
        for (int i = 0; i < SPW; i++)
            if (i < per) {                                   // uniform
                S[r][i] = fmaf(__builtin_amdgcn_exp2f(dt[r] * a[i]), fresh[r] ? 0.f : S[r][i], du * bj[i]);
                y[r] = fmaf(S[r][i], bj[bc_cols + i], y[r]);
            }
    }
    __syncthreads();                                         // everyone has read the sums of dt
#pragma unroll
    for (int r = 0; r < RB; r++) red[wave][r][lane] = y[r];
#pragma unroll
    for (int r = 0; r < RB; r++)
        if (r < rows)
#pragma unroll
            for (int i = 0; i < SPW; i++)
                if (i < per) p.state_out[(b0 + r) * plane + (int64_t)(n0 + i) * g.inner_p + c] = S[r][i];
    __syncthreads();
#pragma unroll
    for (int r = 0; r < RB; r++)
        if (r < rows && wave == (r & 3)) {
            const float t = (red[0][r][lane] + red[1][r][lane]) + (red[2][r][lane] + red[3][r][lane]);
            st_f32((T*)p.out + (int64_t)(b0 + r) * p.ldo + c, fmaf(d, uv[r], t) * silu_f32(zv[r]) * g.out_scale);
        }
}

// MODE WHOLE: all tokens from the stored state, outputs, state out.  SUMS: one chunk from zero, its end and its sum of dt into `ends` /
// `sum_dt`.  OUT: one chunk from its start in `ends`, outputs; the last chunk stores the state.
template <typename T, int SP, int MODE>
__global__ __launch_bounds__(256) void scan_kernel(NcScanGeom g, int lg, const T* __restrict__ u, const float* __restrict__ dt, const float* __restrict__ bc,
                                                   const float* __restrict__ a_log2, const float* __restrict__ skip, const T* __restrict__ z, int ldz,
                                                   const int32_t* __restrict__ seqlens, const float* __restrict__ state_in, float* __restrict__ state_out,
                                                   T* __restrict__ out, int ldo, float* __restrict__ ends, float* __restrict__ sum_dt, int chunks, int chunk_len) {
    extern __shared__ __align__(16) float lds[];            // [TB][2][state_p]: B, C
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, cw = 64 / lg, part = lane / cw;
    const int c_at = ((int)blockIdx.x * 4 + wave) * cw + lane % cw, c = min(c_at, g.inner_p - 1);
    const bool mine = c_at < g.inner_p;
    const int chunk = MODE == SCAN_WHOLE ? 0 : (int)blockIdx.y, b = blockIdx.z;
    const int t_begin = MODE == SCAN_WHOLE ? 0 : chunk * chunk_len, t_end = MODE == SCAN_WHOLE ? g.T : min(g.T, t_begin + chunk_len);
    const int64_t row0 = (int64_t)b * g.T, plane = (int64_t)g.state_p * g.inner_p;
    const int64_t st = (int64_t)b * (g.state_p + g.taps - 1) * g.inner_p + (int64_t)part * SP * g.inner_p + c;
    const int bc_cols = nc_scan_bc_cols(g.state_p);
    float a[SP], S[SP];
#pragma unroll
    for (int i = 0; i < SP; i++) a[i] = a_log2[(int64_t)(part * SP + i) * g.inner_p + c];
    if (MODE == SCAN_SUMS || (chunk == 0 && seqlens[b] == 0)) {
#pragma unroll
        for (int i = 0; i < SP; i++) S[i] = 0.f;
    } else {
        const float* src = MODE == SCAN_OUT && chunk > 0 ? ends + ((int64_t)b * (chunks - 1) + chunk - 1) * plane + (int64_t)part * SP * g.inner_p + c : state_in + st;
#pragma unroll
        for (int i = 0; i < SP; i++) S[i] = src[(int64_t)i * g.inner_p];
    }
    const float d = MODE == SCAN_SUMS ? 0.f : skip[c];
    float total = 0.f;
    for (int t0 = t_begin; t0 < t_end; t0 += TB) {
        float dv[TB], uv[TB], zv[TB];
#pragma unroll
        for (int j = 0; j < TB; j++) {
            const int64_t row = row0 + min(t0 + j, t_end - 1);
            dv[j] = dt[row * g.inner_p + c];
            uv[j] = ld_f32(u + row * g.inner_p + c);
            zv[j] = MODE == SCAN_SUMS ? 0.f : ld_f32(z + row * ldz + c);
        }
        __syncthreads();
        for (int i = 4 * threadIdx.x; i < TB * 2 * g.state_p; i += 1024) {
            const int j = i / (2 * g.state_p), k = i % (2 * g.state_p), which = k / g.state_p;
            *(v4f*)(lds + i) = *(const v4f*)(bc + (row0 + min(t0 + j, t_end - 1)) * 2 * bc_cols + which * bc_cols + k - which * g.state_p);
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < TB; j++) {
            if (t0 + j >= t_end) break;                     // uniform
            const float* bj = lds + j * 2 * g.state_p + part * SP;
            const float* cj = bj + g.state_p;
            const float du = dv[j] * uv[j];
            float y = 0.f;
            if (MODE == SCAN_SUMS) total += dv[j];
#pragma unroll
            for (int i = 0; i < SP; i += 4) {
                const v4f bv = *(const v4f*)(bj + i), cv = MODE == SCAN_SUMS ? v4f{0.f, 0.f, 0.f, 0.f} : *(const v4f*)(cj + i);
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    S[i + r] = fmaf(__builtin_amdgcn_exp2f(dv[j] * a[i + r]), S[i + r], du * bv[r]);
                    if (MODE != SCAN_SUMS) y = fmaf(S[i + r], cv[r], y);
                }
            }
            if (MODE != SCAN_SUMS) {
                for (int o = cw; o < 64; o <<= 1) y += __shfl_xor(y, o);
                y = fmaf(d, uv[j], y) * silu_f32(zv[j]) * g.out_scale;
                if (part == 0 && mine) st_f32(out + (row0 + t0 + j) * ldo + c, y);
            }
        }
    }
    if (!mine) return;
    if (MODE == SCAN_SUMS) {
        float* dst = ends + ((int64_t)b * (chunks - 1) + chunk) * plane + (int64_t)part * SP * g.inner_p + c;
#pragma unroll
        for (int i = 0; i < SP; i++) dst[(int64_t)i * g.inner_p] = S[i];
        if (part == 0) sum_dt[((int64_t)b * (chunks - 1) + chunk) * g.inner_p + c] = total;
    } else if (MODE == SCAN_WHOLE || chunk == chunks - 1) {
#pragma unroll
        for (int i = 0; i < SP; i++) state_out[st + (int64_t)i * g.inner_p] = S[i];
    }
}

// Every chunk's end from a zero state becomes the true start of the next chunk, in place.  One thread per channel and state.
__global__ __launch_bounds__(256) void scan_chunks_kernel(NcScanGeom g, const float* __restrict__ a_log2, const int32_t* __restrict__ seqlens,
                                                          const float* __restrict__ state_in, float* __restrict__ ends, const float* __restrict__ sum_dt, int chunks) {
    const int c = (int)blockIdx.x * 256 + (int)threadIdx.x, n = blockIdx.y, b = blockIdx.z;
    if (c >= g.inner_p) return;
    const int64_t plane = (int64_t)g.state_p * g.inner_p;
    const float a = a_log2[(int64_t)n * g.inner_p + c];
    float S = seqlens[b] > 0 ? state_in[((int64_t)b * (g.state_p + g.taps - 1) + n) * g.inner_p + c] : 0.f;
    float* e = ends + (int64_t)b * (chunks - 1) * plane + (int64_t)n * g.inner_p + c;
    const float* sd = sum_dt + (int64_t)b * (chunks - 1) * g.inner_p + c;
    constexpr int AHEAD = 16;
    for (int k0 = 0; k0 < chunks - 1; k0 += AHEAD) {
        float own[AHEAD], s[AHEAD];
#pragma unroll
        for (int j = 0; j < AHEAD; j++) {
            const int k = min(k0 + j, chunks - 2);
            own[j] = e[k * plane], s[j] = sd[(int64_t)k * g.inner_p];
        }
#pragma unroll
        for (int j = 0; j < AHEAD; j++) {
            if (k0 + j >= chunks - 1) break;
            S = fmaf(__builtin_amdgcn_exp2f(a * s[j]), S, own[j]);
            e[(k0 + j) * plane] = S;
        }
    }
}

constexpr int CHUNK = 64, CHUNK_MIN_TOKENS = 96;
// states per lane and lanes per channel (0: not such a size)
bool lanes_of(int state_p, int& sp, int& lg) {
    for (int s : {16, 12, 8, 4}) {
        const int l = state_p / s;
        if (state_p % s == 0 && (l & (l - 1)) == 0 && l >= 1 && l <= 16) {
            sp = s, lg = l;
            return true;
        }
    }
    return false;
}

int channel_groups(const NcScanGeom& g, int lg) { return (g.inner_p + 4 * (64 / lg) - 1) / (4 * (64 / lg)); }
// Tokens per chunk (0: one pass): at most CHUNK, and so few that the workgroups come out in whole rounds of compute units.
int chunk_len(const NcScanGeom& g) {
    int sp = 0, lg = 0;
    if (g.T < CHUNK_MIN_TOKENS || !lanes_of(g.state_p, sp, lg)) return 0;
    const int per_chunk = channel_groups(g, lg) * g.B, least = (g.T + CHUNK - 1) / CHUNK, cus = nc_cu_count();
    const int64_t rounds = ((int64_t)per_chunk * least + cus - 1) / cus;
    const int chunks = (int)(rounds * cus / per_chunk);
    const int len = ((g.T + chunks - 1) / chunks + TB - 1) / TB * TB;
    return len < 32 ? 32 : len;
}
int chunk_count(const NcScanGeom& g) {
    const int len = chunk_len(g);
    return len ? (g.T + len - 1) / len : 1;
}

template <typename T, int SP>
int launch_scan(const NcScanGeom& g, int lg, const T* u, const float* dt, const float* bc, const float* a_log2, const float* skip, const T* z, int ldz,
                const int32_t* seqlens, const float* state_in, float* state_out, T* out, int ldo, void* workspace, hipStream_t s) {
    const int chunks = chunk_count(g), len = chunk_len(g), xs = channel_groups(g, lg), bytes = TB * 2 * g.state_p * 4;
    if (chunks == 1) {
        hipLaunchKernelGGL((scan_kernel<T, SP, SCAN_WHOLE>), dim3(xs, 1, g.B), dim3(256), bytes, s, g, lg, u, dt, bc, a_log2, skip, z, ldz, seqlens, state_in, state_out,
                           out, ldo, nullptr, nullptr, 1, 0);
        NC_CHECK_LAUNCH("scan");
        return 0;
    }
    float* ends = (float*)workspace;
    float* sum_dt = ends + (int64_t)g.B * (chunks - 1) * g.state_p * g.inner_p;
    hipLaunchKernelGGL((scan_kernel<T, SP, SCAN_SUMS>), dim3(xs, chunks - 1, g.B), dim3(256), bytes, s, g, lg, u, dt, bc, a_log2, skip, z, ldz, seqlens, state_in,
                       state_out, out, ldo, ends, sum_dt, chunks, len);
    hipLaunchKernelGGL(scan_chunks_kernel, dim3((g.inner_p + 255) / 256, g.state_p, g.B), dim3(256), 0, s, g, a_log2, seqlens, state_in, ends, sum_dt, chunks);
    hipLaunchKernelGGL((scan_kernel<T, SP, SCAN_OUT>), dim3(xs, chunks, g.B), dim3(256), bytes, s, g, lg, u, dt, bc, a_log2, skip, z, ldz, seqlens, state_in, state_out,
                       out, ldo, ends, sum_dt, chunks, len);
    NC_CHECK_LAUNCH("scan_chunked");
    return 0;
}
}  // namespace

int nc_launch_scan_conv(int dtype, const NcScanGeom& g, const void* x, int ldx, const float* w, const float* b, const int32_t* seqlens, const float* state_in,
                        float* state_out, void* u, hipStream_t s) {
    NC_CHECK_ARG(x && w && b && u && state_in != state_out && g.taps >= 1 && g.inner_p % 4 == 0 && ldx % 4 == 0, "scan_conv: %d taps, %d channels", g.taps, g.inner_p);
    NC_CHECK_ARG(g.T <= 65535 * CONV_TOKENS && g.B <= 65535, "scan_conv: %d tokens in one portion", g.T);
    NcProfScope prof(NC_CLS_ROWS, (double)g.B * g.T * g.inner_p * (dtype ? 8 : 4), s);
    const dim3 grid((g.inner_p + 1023) / 1024, (g.T + CONV_TOKENS - 1) / CONV_TOKENS, g.B);
    if (dtype)
        hipLaunchKernelGGL((scan_conv_kernel<float>), grid, dim3(256), 0, s, g, (const float*)x, ldx, w, b, seqlens, state_in, state_out, (float*)u);
    else
        hipLaunchKernelGGL((scan_conv_kernel<bf16_t>), grid, dim3(256), 0, s, g, (const bf16_t*)x, ldx, w, b, seqlens, state_in, state_out, (bf16_t*)u);
    NC_CHECK_LAUNCH("scan_conv");
    return 0;
}

int nc_launch_scan_join(int dtype, const NcScanGeom& g, const float* parts, int splits, void* dtr, float* bc, hipStream_t s) {
    const int bc_cols = nc_scan_bc_cols(g.state_p);
    const int64_t M = (int64_t)g.B * g.T, work = M * (g.dt_rank_p + 2 * bc_cols) / 4;
    NC_CHECK_ARG(parts && dtr && bc && splits >= 1 && g.dt_rank_p % 4 == 0, "scan_join: null operand");
    NcProfScope prof(NC_CLS_ROWS, (double)work * 16 * (splits + 1), s);
    if (dtype)
        hipLaunchKernelGGL((scan_join_kernel<float>), dim3((unsigned)((work + 255) / 256)), dim3(256), 0, s, parts, splits, M, g.dt_rank_p, bc_cols, (float*)dtr, bc);
    else
        hipLaunchKernelGGL((scan_join_kernel<bf16_t>), dim3((unsigned)((work + 255) / 256)), dim3(256), 0, s, parts, splits, M, g.dt_rank_p, bc_cols, (bf16_t*)dtr, bc);
    NC_CHECK_LAUNCH("scan_join");
    return 0;
}

int nc_launch_scan_step(int dtype, const NcScanGeom& g, const NcScanStep& p, hipStream_t s) {
    NC_CHECK_ARG(g.T == 1 && g.state_p % 4 == 0 && g.state_p <= 256 && g.inner_p % 64 == 0 && g.dt_rank_p % 64 == 0, "scan_step: %d tokens, %d states", g.T, g.state_p);
    NC_CHECK_ARG(p.parts && p.splits >= 1 && p.w_dt_t && p.dt_b && p.a_log2 && p.skip && p.u && p.z && p.out && p.state_in != p.state_out, "scan_step: null operand");
    const int N = g.dt_rank_p + 2 * nc_scan_bc_cols(g.state_p), per = g.state_p / 4;
    // state in and out, the step's weight once, the rows in and out (bytes)
    const double es = dtype ? 4 : 2;
    NcProfScope prof(NC_CLS_SCAN, (double)g.B * (8.0 * g.state * g.inner + g.inner * 3 * es) + (double)g.dt_rank_p * g.inner * es, s, g.T);
    // (few rows: one each, so that the launch covers the chip)
    const int rb = per <= 16 && (int64_t)g.B * (g.inner_p / 64) >= 4 * nc_cu_count() ? 4 : 1;
    const int bytes = rb * N * 4;
    NC_CHECK_ARG(bytes <= 56 * 1024 && (g.B + rb - 1) / rb <= 65535, "scan_step: a step of rank %d", g.dt_rank_p);
    const dim3 grid(g.inner_p / 64, (g.B + rb - 1) / rb);
#define GO(RB, SPW)                                                                                          \
    do {                                                                                                     \
        if (dtype) hipLaunchKernelGGL((scan_step_kernel<float, RB, SPW>), grid, dim3(256), bytes, s, g, p);  \
        else hipLaunchKernelGGL((scan_step_kernel<bf16_t, RB, SPW>), grid, dim3(256), bytes, s, g, p);       \
    } while (0)
    if (rb == 4) {
        if (per <= 4) GO(4, 4);
        else if (per <= 8) GO(4, 8);
        else GO(4, 16);
    } else {
        if (per <= 4) GO(1, 4);
        else if (per <= 16) GO(1, 16);
        else GO(1, 64);
    }
#undef GO
    NC_CHECK_LAUNCH("scan_step");
    return 0;
}

size_t nc_scan_workspace_bytes(const NcScanGeom& g) {
    const int chunks = chunk_count(g);
    return chunks > 1 ? (size_t)g.B * (chunks - 1) * (g.state_p + 1) * g.inner_p * sizeof(float) : 0;
}

int nc_launch_scan(int dtype, const NcScanGeom& g, const void* u, const float* dt, const float* bc, const float* a_log2, const float* skip, const void* z, int ldz,
                   const int32_t* seqlens, const float* state_in, float* state_out, void* out, int ldo, void* workspace, hipStream_t s) {
    int sp = 0, lg = 0;
    NC_CHECK_ARG(lanes_of(g.state_p, sp, lg) && g.state <= g.state_p, "scan: %d states per channel in %d", g.state, g.state_p);
    NC_CHECK_ARG(u && dt && bc && a_log2 && skip && z && out && state_in != state_out, "scan: null operand");
    NC_CHECK_ARG(g.T <= 65535 * 32 && g.B <= 65535, "scan: %d tokens in one portion", g.T);
    // state in and out once; per token the projections and the result (bytes)
    NcProfScope prof(NC_CLS_SCAN, (double)g.B * (8.0 * g.state * g.inner_p + (double)g.T * g.inner_p * (4 + (dtype ? 12 : 6))), s, g.T);
#define GO(SP)                                                                                                                                           \
    (dtype ? launch_scan<float, SP>(g, lg, (const float*)u, dt, bc, a_log2, skip, (const float*)z, ldz, seqlens, state_in, state_out, (float*)out, ldo,   \
                                    workspace, s)                                                                                                         \
           : launch_scan<bf16_t, SP>(g, lg, (const bf16_t*)u, dt, bc, a_log2, skip, (const bf16_t*)z, ldz, seqlens, state_in, state_out, (bf16_t*)out, ldo, \
                                     workspace, s))
    switch (sp) {
        case 16: return GO(16);
        case 12: return GO(12);
        case 8: return GO(8);
        default: return GO(4);
    }
#undef GO
}
