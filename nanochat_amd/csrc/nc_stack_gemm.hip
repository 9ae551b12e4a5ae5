// Linears of the layer stack:  out[M,N] = A[M,K] . W[N,K]^T  on the matrix cores, bfloat16 (v_mfma_f32_16x16x32_bf16) or true 32-bit
// (v_mfma_f32_16x16x4_f32) operands, 32-bit sums.  Both formats share one data path counted in bytes: a lane supplies 16 bytes of row
// (lane & 15) from K-piece (lane >> 4), which is one bf16 instruction or four fp32 ones -- which k a lane's bytes stand for does not
// matter as long as both operands agree.  Operands are issued as (W, A), so a lane ends up with four consecutive output columns of
// one output row.
//
//   linear_few_kernel    up to 64 rows (decode): the weight is streamed once, K is dealt to the four waves of a workgroup (and, where a
//                        consumer adds partial sums, to several workgroups); no LDS in the loop.
//   linear_tiled_kernel  more rows: 64 x 128 or 128 x 256 tiles, operands straight into a ring of three LDS stages.
//
// A stacked weight is several matrices that read the same input; the epilogue sends each run of output columns its own way (store,
// gelu, silu, GLUs, softplus, router logits, residual add, soft-capped logits).  Rows can be grouped by weight (experts).
#include <atomic>
#include "nc_stack.h"

typedef __bf16 v8bf __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) void* lds_ptr_t;

namespace {
template <typename T> struct Mma;
template <> struct Mma<bf16_t> {
    static __device__ __forceinline__ v4f run(const v4i& w, const v4i& a, const v4f& c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(v8bf, w), __builtin_bit_cast(v8bf, a), c, 0, 0, 0);
    }
};
template <> struct Mma<float> {
    static __device__ __forceinline__ v4f run(const v4i& w, const v4i& a, const v4f& c) {
        const v4f wf = __builtin_bit_cast(v4f, w), af = __builtin_bit_cast(v4f, a);
        v4f r = c;
#pragma unroll
        for (int j = 0; j < 4; j++) r = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[j], af[j], r, 0, 0, 0);
        return r;
    }
};

// One instruction of the same, accumulated in place and kept in program order against every memory operation: the builtin lets the register
// allocator pick another result tuple, which it repairs with copies in every K-step, and nothing would keep the LDS reads of a step in
// front of the barrier that ends it.  PARTS instructions make up 16 bytes; the caller puts other accumulators between them.
template <typename T> constexpr int MMA_PARTS = sizeof(T) == 2 ? 1 : 4;
template <typename T>
__device__ __forceinline__ void mma_in_place(v4f& acc, const v4i& w, const v4i& a, int part) {
    if constexpr (sizeof(T) == 2) asm volatile("v_mfma_f32_16x16x32_bf16 %0, %1, %2, %0" : "+a"(acc) : "v"(w), "v"(a) : "memory");
    else asm volatile("v_mfma_f32_16x16x4_f32 %0, %1, %2, %0" : "+a"(acc) : "v"(w[part]), "v"(a[part]) : "memory");
}

// four consecutive columns n .. n+3 (n a multiple of 4, all in one segment) of output row `row`
template <typename T>
__device__ __forceinline__ void store_cols(const NcLinear& g, int64_t out_off, int row, int n, v4f v) {
    int s = 0, base = 0;
#pragma unroll
    for (int i = 0; i < 3; i++)
        if (i + 1 < g.nseg && n >= g.seg[i].end) s = i + 1, base = g.seg[i].end;
    const NcSeg sg = g.seg[s];
    const int c = n - base;
    switch (sg.kind) {
        case NC_SEG_PLAIN: st4_f32((T*)sg.out + out_off + (int64_t)row * sg.ld + c, v); break;
        case NC_SEG_GELU:
            st4_f32((T*)sg.out + out_off + (int64_t)row * sg.ld + c,
                    v4f{gelu_tanh_f32(v[0]), gelu_tanh_f32(v[1]), gelu_tanh_f32(v[2]), gelu_tanh_f32(v[3])});
            break;
        case NC_SEG_GLU: {
            T* o = (T*)sg.out + out_off + (int64_t)row * sg.ld + (c >> 1);
            const float y0 = clamped_glu_f32(v[0], v[1], sg.p0), y1 = clamped_glu_f32(v[2], v[3], sg.p0);
            if constexpr (sizeof(T) == 2) *(uint32_t*)o = pack_bf16(y0, y1);
            else o[0] = y0, o[1] = y1;
            break;
        }
        case NC_SEG_SILU: st4_f32((T*)sg.out + out_off + (int64_t)row * sg.ld + c, v4f{silu_f32(v[0]), silu_f32(v[1]), silu_f32(v[2]), silu_f32(v[3])}); break;
        case NC_SEG_SWIGLU: {
            T* o = (T*)sg.out + out_off + (int64_t)row * sg.ld + (c >> 1);
            const float y0 = silu_f32(v[0]) * v[1], y1 = silu_f32(v[2]) * v[3];
            if constexpr (sizeof(T) == 2) *(uint32_t*)o = pack_bf16(y0, y1);
            else o[0] = y0, o[1] = y1;
            break;
        }
        case NC_SEG_SOFTPLUS: {
            const v4f z = v + *(const v4f*)(sg.bias + c);
            *(v4f*)((float*)sg.out + out_off + (int64_t)row * sg.ld + c) = v4f{softplus_f32(z[0]), softplus_f32(z[1]), softplus_f32(z[2]), softplus_f32(z[3])};
            break;
        }
        case NC_SEG_F32: *(v4f*)((float*)sg.out + out_off + (int64_t)row * sg.ld + c) = v; break;
        case NC_SEG_RESIDUAL: {
            v4f* o = (v4f*)((float*)sg.out + out_off + (int64_t)row * sg.ld + c);
            *o = *o + v;
            break;
        }
        default: {
            float* o = (float*)sg.out + out_off + (int64_t)row * sg.ld + c;
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (n + r < g.N) {
                    const float z = v[r] * sg.p0;
                    o[r] = sg.p1 > 0.f ? sg.p1 * tanhf(z / sg.p1) : z;
                }
        }
    }
}

// What a workgroup works on: which rows of A, which weight, where the output starts.
struct Span {
    int row0, rows;          // output rows [row0, row0 + rows)
    int64_t a_off, w_off, out_off;
};
__device__ __forceinline__ bool find_span(const NcLinear& g, int y, int batch, int tile_rows, Span& sp) {
    if (g.tiles) {
        if (y >= *g.n_tiles) return false;
        const int32_t* t = g.tiles + NC_TILE_WORDS * y;
        sp = Span{t[1], t[2], 0, (int64_t)t[0] * g.w_stride, 0};
        return true;
    }
    sp = Span{y * tile_rows, min(g.M - y * tile_rows, tile_rows), batch * g.a_stride, batch * g.w_stride, batch * g.out_stride};
    return sp.rows > 0;
}
__device__ __forceinline__ int64_t a_row(const NcLinear& g, int row) { return g.a_rows ? g.a_rows[row] / g.a_div : row; }

// ------------------------------------------------------------------------------------------------
// MT tiles of 16 rows x NB tiles of 16 weight rows per workgroup; wave w takes K-steps [its share] of 64 bytes.
template <typename T, int MT, int NB>
__global__ __launch_bounds__(256) void linear_few_kernel(NcLinear g) {
    __shared__ v4f red[4][MT * NB][64];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int split = (int)blockIdx.z % g.splits, batch = (int)blockIdx.z / g.splits;
    Span sp;
    if (!find_span(g, blockIdx.y, batch, 16 * MT, sp)) return;
    const int n0 = blockIdx.x * 16 * NB, frow = lane & 15, piece = lane >> 4;
    const uint8_t* wp[NB];
    const uint8_t* ap[MT];
#pragma unroll
    for (int j = 0; j < NB; j++) {
        const int n = min(n0 + 16 * j + frow, g.N - 1);
        wp[j] = (const uint8_t*)((const T*)g.w + sp.w_off + (int64_t)n * g.ldw) + piece * 16;
    }
#pragma unroll
    for (int i = 0; i < MT; i++) {
        const int m = sp.row0 + min(16 * i + frow, sp.rows - 1);
        ap[i] = (const uint8_t*)((const T*)g.a + sp.a_off + a_row(g, m) * g.lda) + piece * 16;
    }
    v4f acc[MT][NB];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < NB; j++) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};

    const int steps = g.K * (int)sizeof(T) / 64, shares = 4 * g.splits, share = 4 * split + wave;
    const int s0 = (int)((int64_t)steps * share / shares), s1 = (int)((int64_t)steps * (share + 1) / shares);
    constexpr int U = MT * NB >= 16 ? 2 : 4;
    auto step = [&](int s, auto unroll) {
        constexpr int N_ = decltype(unroll)::value;
        v4i wf[N_][NB], af[N_][MT];
#pragma unroll
        for (int u = 0; u < N_; u++) {
#pragma unroll
            for (int j = 0; j < NB; j++) wf[u][j] = __builtin_nontemporal_load((const v4i*)(wp[j] + (int64_t)(s + u) * 64));
#pragma unroll
            for (int i = 0; i < MT; i++) af[u][i] = *(const v4i*)(ap[i] + (int64_t)(s + u) * 64);
        }
#pragma unroll
        for (int u = 0; u < N_; u++)
#pragma unroll
            for (int j = 0; j < NB; j++)
#pragma unroll
                for (int i = 0; i < MT; i++) acc[i][j] = Mma<T>::run(wf[u][j], af[u][i], acc[i][j]);
    };
    int s = s0;
    for (; s + U <= s1; s += U) step(s, std::integral_constant<int, U>{});
    for (; s < s1; s++) step(s, std::integral_constant<int, 1>{});

#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < NB; j++) red[wave][i * NB + j][lane] = acc[i][j];
    __syncthreads();
    for (int t = wave; t < MT * NB; t += 4) {
        const int i = t / NB, j = t % NB;
        const int m = 16 * i + frow, n = n0 + 16 * j + 4 * piece;
        if (m >= sp.rows || n >= g.N) continue;
        const v4f v = (red[0][t][lane] + red[1][t][lane]) + (red[2][t][lane] + red[3][t][lane]);
        if (g.partials) *(v4f*)(g.partials + ((int64_t)split * g.M + sp.row0 + m) * g.N + n) = v;
        else store_cols<T>(g, sp.out_off, sp.row0 + m, n, v);
    }
}

// ------------------------------------------------------------------------------------------------
// BM x BN outputs, WM x WN waves of 16-row, 16-column tiles, K-steps of 128 bytes.  Operand tiles go from global memory straight into LDS,
// 1 KB (8 rows x 128 bytes) per load instruction; chunk c (16 bytes) of row r is kept at slot c ^ SWZ(r), the permutation being applied
// on the global side, so that the fragment reads of 16 rows are free of bank conflicts.  A ring of STAGES: the loads of STAGES - 1 steps
// are in flight while one is multiplied.  Past the end of K the loads are issued all the same (into stages nobody reads any more), so
// that the barrier counts the same number of loads in every step.
#define TILE_SWZ(row) (((row) & 7) ^ (((row) >> 3) & 1))
#define TILE_OOB 0x80000000u       // a buffer offset past every descriptor: the load returns zeros
#define TILE_GROUP_M 8

// Tile order: workgroups are dealt to the 8 XCDs (each with an L2 of its own) in turn, so every XCD gets a contiguous run of the
// sequence, and the sequence walks bands of TILE_GROUP_M tile rows column by column.
__device__ __forceinline__ void tile_order(int id, int tiles_m, int tiles_n, int& tm, int& tn) {
    const int total = tiles_m * tiles_n, xcd = id & 7, slot = id >> 3;
    const int lin = xcd * (total >> 3) + min(xcd, total & 7) + slot;
    const int band = TILE_GROUP_M * tiles_n, first = (lin / band) * TILE_GROUP_M, rows = min(TILE_GROUP_M, tiles_m - first);
    tm = first + (lin % band) % rows, tn = (lin % band) / rows;
}

// Grouped rows: every XCD gets a contiguous run of (group, column tile, row tile of the group), the row tiles innermost, so that a weight
// tile is read by neighbours.  The launch covers the most tiles there can be; those past the actual count leave.
__device__ __forceinline__ bool group_tile_order(const NcLinear& g, int id, int tiles_n, int& tm, int& tn) {
    const int total = *g.n_tiles * tiles_n;
    if (id >= total) return false;
    const int xcd = id & 7, lin = xcd * (total >> 3) + min(xcd, total & 7) + (id >> 3);
    const int32_t* t = g.tiles + NC_TILE_WORDS * (lin / tiles_n);
    const int first = t[3], count = t[4], o = lin - first * tiles_n;
    tm = first + o % count, tn = o / count;
    return true;
}

template <int A_P, int W_P, int STRIDE>
__device__ __forceinline__ void tile_fetch(const void* A, uint32_t a_bytes, const void* W, uint32_t w_bytes, uint8_t* st, int w_part,
                                           const uint32_t* vo_a, const uint32_t* vo_w, int k_off) {
    const __amdgpu_buffer_rsrc_t da = __builtin_amdgcn_make_buffer_rsrc((void*)A, 0, a_bytes, 0x00020000);
    const __amdgpu_buffer_rsrc_t dw = __builtin_amdgcn_make_buffer_rsrc((void*)W, 0, w_bytes, 0x00020000);
#pragma unroll
    for (int i = 0; i < A_P; i++) __builtin_amdgcn_raw_ptr_buffer_load_lds(da, (lds_ptr_t)(st + i * STRIDE), 16, vo_a[i], k_off, 0, 0);
#pragma unroll
    for (int i = 0; i < W_P; i++) __builtin_amdgcn_raw_ptr_buffer_load_lds(dw, (lds_ptr_t)(st + w_part + i * STRIDE), 16, vo_w[i], k_off, 0, 0);
}

template <typename T, int BM, int BN, int WM, int WN, int STAGES>
__global__ __launch_bounds__(64 * WM * WN) void linear_tiled_kernel(NcLinear g, int tiles_m, int tiles_n, uint32_t a_bytes) {
    constexpr int NW = WM * WN, WTM = BM / WM / 16, WTN = BN / WN / 16, STAGE = (BM + BN) * 128, A_P = BM / 8 / NW, W_P = BN / 8 / NW;
    // s_waitcnt vmcnt(loads of the STAGES - 2 youngest steps), other counters untouched
    constexpr int FLIGHT = (STAGES - 2) * (A_P + W_P), WAIT = 0x0F70 | (FLIGHT & 15) | ((FLIGHT >> 4) << 14);
    static_assert(A_P >= 1 && W_P >= 1 && NW % 2 == 0, "waves");
    extern __shared__ __align__(16) uint8_t lds[];
    int tm, tn;
    if (g.tiles) {
        if (!group_tile_order(g, blockIdx.x, tiles_n, tm, tn)) return;
    } else {
        tile_order(blockIdx.x, tiles_m, tiles_n, tm, tn);
    }
    Span sp;
    if (!find_span(g, tm, blockIdx.y, BM, sp)) return;
    const int n0 = tn * BN;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int wm = wave / WN, wn = wave % WN, frow = lane & 15, piece = lane >> 4;
    // staging: piece i of this wave is the 1 KB block (wave + NW i) of its operand's part of the stage; this lane's row inside an 8-row
    // block, and the global chunk that belongs in its LDS slot
    const int sub = lane >> 3, gch = (lane & 7) ^ sub ^ (wave & 1);
    const int rd_lo = frow * 128 + (((2 * piece) ^ TILE_SWZ(frow)) << 4), rd_hi = frow * 128 + (((2 * piece + 1) ^ TILE_SWZ(frow)) << 4);
    const uint32_t row_a = (uint32_t)(g.lda * sizeof(T)), row_w = (uint32_t)(g.ldw * sizeof(T)), k_bytes = (uint32_t)(g.K * sizeof(T));
    const T* const A = (const T*)g.a + sp.a_off;
    const T* const W = (const T*)g.w + sp.w_off;
    uint32_t vo_a[A_P], vo_w[W_P];
#pragma unroll
    for (int i = 0; i < A_P; i++) {
        const int r = 8 * (wave + NW * i) + sub;
        vo_a[i] = r < sp.rows ? (uint32_t)a_row(g, sp.row0 + r) * row_a + gch * 16 : TILE_OOB;
    }
#pragma unroll
    for (int i = 0; i < W_P; i++) {
        const int r = n0 + 8 * (wave + NW * i) + sub;
        vo_w[i] = r < g.N ? (uint32_t)r * row_w + gch * 16 : TILE_OOB;
    }
    const int ksteps = k_bytes / 128;
    v4f acc[WTM][WTN];
#pragma unroll
    for (int i = 0; i < WTM; i++)
#pragma unroll
        for (int j = 0; j < WTN; j++) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};
    auto fetch = [&](int t, int stage) {
        tile_fetch<A_P, W_P, NW * 1024>(A, a_bytes, W, (uint32_t)(g.N - 1) * row_w + k_bytes, lds + stage * STAGE + wave * 1024, BM * 128, vo_a, vo_w,
                                        t < ksteps ? t * 128 : 0);
    };
    auto meet = [&]() {
        asm volatile("" ::: "memory");
        __builtin_amdgcn_s_waitcnt(WAIT);    // the operands of the next step have landed (this wave's share; the barrier says everybody's)
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
    };
#pragma unroll
    for (int i = 0; i < STAGES - 1; i++) fetch(i, i);
    meet();
    int cur = 0, nxt = STAGES - 1;
    for (int kt = 0; kt < ksteps; kt++) {
        const uint8_t* a = lds + cur * STAGE + wm * (BM / WM) * 128;
        const uint8_t* w = lds + cur * STAGE + BM * 128 + wn * (BN / WN) * 128;
        v4i al[WTM], ah[WTM], wl[2], wh[2];
        wl[0] = *(const v4i*)(w + rd_lo);
#pragma unroll
        for (int i = 0; i < WTM; i++) al[i] = *(const v4i*)(a + i * 2048 + rd_lo);
        wh[0] = *(const v4i*)(w + rd_hi);
#pragma unroll
        for (int i = 0; i < WTM; i++) ah[i] = *(const v4i*)(a + i * 2048 + rd_hi);
        fetch(kt + STAGES - 1, nxt);         // into the stage read in step kt - 1: everyone is past the barrier that ended it
#pragma unroll
        for (int j = 0; j < WTN; j++) {
            if (j + 1 < WTN) {               // one group ahead of its use
                wl[(j + 1) & 1] = *(const v4i*)(w + (j + 1) * 2048 + rd_lo);
                wh[(j + 1) & 1] = *(const v4i*)(w + (j + 1) * 2048 + rd_hi);
            }
#pragma unroll
            for (int p = 0; p < MMA_PARTS<T>; p++)
#pragma unroll
                for (int i = 0; i < WTM; i++) mma_in_place<T>(acc[i][j], wl[j & 1], al[i], p);
#pragma unroll
            for (int p = 0; p < MMA_PARTS<T>; p++)
#pragma unroll
                for (int i = 0; i < WTM; i++) mma_in_place<T>(acc[i][j], wh[j & 1], ah[i], p);
        }
        meet();
        cur = cur + 1 == STAGES ? 0 : cur + 1;
        nxt = nxt + 1 == STAGES ? 0 : nxt + 1;
    }
    // the loads past the end of K are still landing: they must be done before the workgroup gives its LDS back
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_waitcnt(0x0F70);
    __builtin_amdgcn_s_barrier();
    // (the last products: the compiler does not see that an asm statement wrote the accumulators late)
    asm volatile("s_nop 15\n\ts_nop 15" ::: "memory");
#pragma unroll
    for (int i = 0; i < WTM; i++)
#pragma unroll
        for (int j = 0; j < WTN; j++) asm volatile("" : "+a"(acc[i][j]));
#pragma unroll
    for (int i = 0; i < WTM; i++) {
        const int m = wm * (BM / WM) + 16 * i + frow;
        if (m >= sp.rows) continue;
#pragma unroll
        for (int j = 0; j < WTN; j++) {
            const int n = n0 + wn * (BN / WN) + 16 * j + 4 * piece;
            if (n < g.N) store_cols<T>(g, sp.out_off, sp.row0 + m, n, acc[i][j]);
        }
    }
}

int reserve_dynamic_lds(const void* fn, int bytes, std::atomic<uint64_t>& done) {
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev > 63) dev = 0;
    if (done.load(std::memory_order_relaxed) >> dev & 1) return 0;
    if (hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) != hipSuccess) NC_FAIL(-2, "linear: %d bytes of LDS refused", bytes);
    done.fetch_or(1ull << dev, std::memory_order_relaxed);
    return 0;
}

int check_linear(const NcLinear& l, int dtype) {
    NC_CHECK_ARG(l.a && l.w && l.nseg <= 4, "linear: null operand");
    NC_CHECK_ARG(l.M > 0 && l.N > 0 && l.K > 0 && l.K % 32 == 0 && l.batch >= 1, "linear: bad shape M=%d N=%d K=%d batch=%d", l.M, l.N, l.K, l.batch);
    NC_CHECK_ARG(dtype == 0 || dtype == 1, "linear: dtype must be 0 (bfloat16) or 1 (float)");
    NC_CHECK_ARG(l.lda % (dtype ? 4 : 8) == 0 && l.ldw % (dtype ? 4 : 8) == 0 && l.ldw >= l.K && ((uintptr_t)l.a & 15) == 0 && ((uintptr_t)l.w & 15) == 0, "linear: operands must be 16-byte aligned");
    for (int i = 0; i < l.nseg; i++)
        NC_CHECK_ARG(l.seg[i].kind == NC_SEG_LOGITS || (l.seg[i].end % 16 == 0 && l.seg[i].ld % 4 == 0), "linear: segments must end at multiples of 16 columns");
    return 0;
}

template <typename T, int MT, int NB>
int launch_few(const NcLinear& l, int ytiles, hipStream_t s) {
    hipLaunchKernelGGL((linear_few_kernel<T, MT, NB>), dim3((l.N + 16 * NB - 1) / (16 * NB), ytiles, l.batch * l.splits), dim3(256), 0, s, l);
    NC_CHECK_LAUNCH("linear_few");
    return 0;
}
template <typename T>
int launch_few_t(const NcLinear& l, hipStream_t s) {
    if (l.tiles) return l.N >= 2048 ? launch_few<T, 1, 2>(l, l.max_tiles, s) : launch_few<T, 1, 1>(l, l.max_tiles, s);
    if (l.M <= 16) return (int64_t)l.N * l.splits * l.batch >= 16384 ? launch_few<T, 1, 2>(l, 1, s) : launch_few<T, 1, 1>(l, 1, s);
    if (l.M <= 32) return launch_few<T, 2, 2>(l, 1, s);
    // (64 rows, K = 2048: N = 32768 54 us with four column tiles per workgroup against 66 with two, N = 7808 32 against 19)
    return l.N >= 16384 ? launch_few<T, 4, 4>(l, (l.M + 63) / 64, s) : launch_few<T, 4, 2>(l, (l.M + 63) / 64, s);
}
template <typename T, int BM, int BN, int WM, int WN, int STAGES>
int launch_tiled(const NcLinear& l, hipStream_t s) {
    static std::atomic<uint64_t> done{0};
    constexpr int LDS = (BM + BN) * 128 * STAGES;
    const void* fn = (const void*)linear_tiled_kernel<T, BM, BN, WM, WN, STAGES>;
    if (int rc = reserve_dynamic_lds(fn, LDS, done)) return rc;
    const int tm = l.tiles ? l.max_tiles : (l.M + BM - 1) / BM, tn = (l.N + BN - 1) / BN;
    // rows of A this launch may reach: all of them (a gathered row index is below M / a_div)
    const int64_t a_rows = l.a_rows ? (l.M + l.a_div - 1) / l.a_div : l.M;
    const int64_t a_bytes = ((a_rows - 1) * l.lda + l.K) * (int64_t)sizeof(T);
    NC_CHECK_ARG(a_bytes < (1ll << 31) && (int64_t)l.N * l.ldw * (int64_t)sizeof(T) < (1ll << 31), "linear: operand past 2 GiB");
    hipLaunchKernelGGL((linear_tiled_kernel<T, BM, BN, WM, WN, STAGES>), dim3(tm * tn, l.batch), dim3(64 * WM * WN), LDS, s, l, tm, tn, (uint32_t)a_bytes);
    NC_CHECK_LAUNCH("linear_tiled");
    return 0;
}
// tile shapes: 1 = 64 x 128 (two workgroups per compute unit), 2 = 128 x 256.  Measured and not kept: 128 x 128 in two stages (711 to 848
// TFLOP/s where 128 x 256 has 833 to 870), 256 x 256 in two stages (598 to 690).
template <typename T>
int launch_tiled_shape(const NcLinear& l, int shape, hipStream_t s) {
    return shape == 1 ? launch_tiled<T, 64, 128, 2, 2, 3>(l, s) : launch_tiled<T, 128, 256, 2, 4, 3>(l, s);
}

double linear_units(const NcLinear& l, int dtype, bool few) {
    // the few-rows kernel is a stream of the weight (bytes), the tiled one a product (flops)
    return few ? (double)l.batch * l.N * l.K * (dtype ? 4 : 2) : 2.0 * l.batch * l.M * l.N * l.K;
}
int64_t linear_tag(const NcLinear& l) { return ((int64_t)l.N << 32) | (uint32_t)l.K; }
}  // namespace

int nc_linear_few_splits(int M, int N, int K) {
    const int nb = M <= 16 ? 16 : 32;
    const int wgs = (N + nb - 1) / nb;
    int splits = 1;
    while (splits < 8 && wgs * splits < 384 && K / (splits * 2) >= 256) splits *= 2;
    return splits;
}

int nc_launch_linear_few(int dtype, const NcLinear& l, hipStream_t s, int cls) {
    if (int rc = check_linear(l, dtype)) return rc;
    NC_CHECK_ARG(!l.tiles || l.tile_rows == NC_GROUP_TILE_FEW, "linear: group tiles of %d rows", l.tile_rows);
    NC_CHECK_ARG(l.splits >= 1 && (l.splits == 1 || l.partials), "linear: split sums need a buffer");
    NcProfScope prof(cls, linear_units(l, dtype, true), s, linear_tag(l));
    return dtype ? launch_few_t<float>(l, s) : launch_few_t<bf16_t>(l, s);
}

int nc_launch_linear_tiled(int dtype, const NcLinear& l, hipStream_t s, int cls, int shape) {
    if (int rc = check_linear(l, dtype)) return rc;
    NC_CHECK_ARG(!l.partials && l.K % 64 == 0, "linear: the tiled kernel takes whole K-steps and finishes its sums");
    NcProfScope prof(cls, linear_units(l, dtype, false), s, linear_tag(l));
    if (!shape) {
        // the widest tile unless it leaves compute units without one (measured at 1792 rows: 858 against 679 TFLOP/s at N = 12352, 551
        // against 717 at N = 2048, where the launch has 112 or 448 tiles)
        const int64_t wide = (int64_t)((l.M + 127) / 128) * ((l.N + 255) / 256) * l.batch;
        // (a sum of a few K-steps is mostly its epilogue: two workgroups per compute unit, one of which works while the other stores)
        const bool brief = l.K * (dtype ? 4 : 2) <= 512;
        shape = l.tiles ? (l.tile_rows == 64 ? 1 : 2) : wide < 200 || brief ? 1 : 2;
    }
    if (l.tiles) NC_CHECK_ARG(l.tile_rows == (shape == 1 ? 64 : 128), "linear: group tiles of %d rows", l.tile_rows);
    return dtype ? launch_tiled_shape<float>(l, shape, s) : launch_tiled_shape<bf16_t>(l, shape, s);
}
