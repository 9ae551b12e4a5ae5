// Host-side sequencing of one forward of the layer stack on a stream (include/nanochat_amd_stack.h): one call enqueues every kernel of
// the step; no host synchronisation, no allocation.
//
// Per run of a parallel layer, h = the normed rows:
//   linear   [projections | router logits | first feed-forward matrix] . h    the activation of the feed-forward in the epilogue
//   mixer    -> its part of `cat`; the feed-forward's part is there already
//   experts  route (softmax, choice, expert order), gate and up with their activation, down: one row per (token, choice)
//   linear   w_out . cat, added to the residual stream: in its epilogue, or (few rows) as partial sums by the row kernel
//   row add  x += partial sums + weighted expert rows (+ embedding output + step vector at the start of a pass), norm -> h
// Per run of a post-norm layer, h = x in the storage type:
//   linear   projections . h;  mixers, side by side if there are two  -> `cat`
//   linear   w_out . cat -> sums in fp32 (few rows: partial ones);  row add  x += norm1(sums) -> h
//   linear   gate and up . h, activation in the epilogue;  linear  down -> sums;  row add  x += norm2(sums) -> h
// Few rows (decode): weights are streamed by linear_few_kernel; more rows: the tiled kernel.
#include "../../include/nanochat_amd_stack.h"
#include "nc_stack.h"

#define TRY(call)              \
    do {                       \
        int rc__ = (call);     \
        if (rc__) return rc__; \
    } while (0)

namespace {
struct Carver {
    uint8_t* base;
    size_t off = 0;
    explicit Carver(void* p) : base((uint8_t*)p) {}
    void* take(size_t bytes) {
        off = (off + 255) & ~(size_t)255;
        void* r = base ? base + off : nullptr;
        off += bytes;
        return r;
    }
};

struct Workspace {
    float *x, *x0, *router, *parts, *raw, *bc, *dt, *x_parts;
    void *h, *proj, *cat, *h_last, *q_lat, *o_lat, *kv, *att_parts, *ret, *act, *e_out, *u, *dtr;
    float* slot_w;
    int32_t *chosen, *slot_of, *perm, *tiles, *n_tiles;
    size_t att_part_bytes, part_bytes, total;
};

NcLatentGeom latent_geom(const nc_stack_mixer& l, int B, int T, int Tmax, int pos_max) {
    return NcLatentGeom{l.heads, l.dim_p, l.rot_p, l.rot_dims, l.rank, l.rank_p, l.vdim_p, l.score_scale, B, T, Tmax, pos_max};
}
NcRetentionGeom retention_geom(const nc_stack_mixer& l, int B, int T, float* raw) {
    return NcRetentionGeom{l.heads, l.dim, l.dim_p, l.vdim, l.vdim_p, l.rot_dims, l.score_scale, B, T, raw};
}
NcWindowGeom window_geom(const nc_stack_mixer& l, int B, int T, int Tmax, int pos_max) {
    return NcWindowGeom{l.heads, l.kv_heads, l.dim, l.dim_p, l.vdim_p, l.rot_dims, l.window, l.keep_first, l.score_scale, l.out_scale, B, T, Tmax, pos_max};
}
// shares of the sum over channels that the few columns of w_x are cut into, to fill the chip
int scan_x_cols(const nc_stack_mixer& l) { return l.dt_rank_p + 2 * nc_scan_bc_cols(l.state_p); }
int scan_x_splits(const nc_stack_mixer& l, int M) {
    if (M <= NC_FEW_ROWS) return nc_linear_few_splits(M, scan_x_cols(l), l.inner_p);
    const int64_t tiles = (int64_t)((M + 63) / 64) * ((scan_x_cols(l) + 127) / 128);
    int splits = 1;
    while (splits < 16 && tiles * splits < 512 && l.inner_p % (2 * splits * NC_STACK_PAD) == 0 && l.inner_p / (2 * splits) >= 256) splits *= 2;
    return splits;
}
NcScanGeom scan_geom(const nc_stack_mixer& l, int B, int T) {
    return NcScanGeom{l.inner, l.inner_p, l.state, l.state_p, l.taps, l.dt_rank_p, l.out_scale, B, T};
}
// Expanding keys and values costs rank (dim + vdim) per key and head; after that a (query, key) pair costs dim + rot + vdim and only the
// visible half of the new pairs is visited, against 2 rank + rot in latent space.
bool expand(int dtype, const nc_stack_mixer& l, const NcLatentGeom& g) {
    if (!nc_latent_expanded_ok(dtype, g) || g.T < 32) return false;
    return (double)g.T * (2.0 * l.rank_p + l.rot_p - 0.5 * (l.dim_p + l.rot_p + l.vdim_p)) > (double)l.rank_p * (l.dim_p + l.vdim_p);
}
int expert_tile_rows(const nc_stack_layer& l, int M) {
    const int per = M * l.top / l.experts;
    return M <= NC_FEW_ROWS || per < 16 ? NC_GROUP_TILE_FEW : per < 128 ? 64 : 128;
}
int expert_max_tiles(const nc_stack_layer& l, int M, int tile_rows) {
    const int pairs = M * l.top;
    return pairs / tile_rows + (pairs < l.experts ? pairs : l.experts);
}
size_t max_of(size_t a, size_t b) { return a > b ? a : b; }

Workspace carve(const nc_stack_model* m, int B, int T, int n_logits, int max_keys, void* base) {
    const size_t M = (size_t)B * T, Wp = m->width_p, es = m->dtype ? 4 : 2;
    size_t proj = 0, router = 0, parts = 0, qlat = 0, olat = 0, kv = 0, att = 0, ret = 0, act = 0, eout = 0, pairs = 0, tiles = 0, raw = 0, bc = 0, dt = 0, u = 0,
           dtr = 0, x_parts = 0;
    bool again = false;
    for (int i = 0; i < m->n_runs; i++) again |= m->runs[i].add_embedding != 0;
    for (int i = 0; i < m->n_layers; i++) {
        const nc_stack_layer& l = m->layers[i];
        proj = max_of(proj, M * l.mix_cols * es);
        router = max_of(router, M * l.router_cols * 4);
        if (M <= NC_FEW_ROWS) parts = max_of(parts, (size_t)nc_linear_few_splits((int)M, (int)Wp, l.k_out) * M * Wp * 4);
        else if (l.block == NC_BLOCK_POST_NORM) parts = max_of(parts, M * Wp * 4);
        if (l.block == NC_BLOCK_POST_NORM && l.ff) {
            if (M <= NC_FEW_ROWS) parts = max_of(parts, (size_t)nc_linear_few_splits((int)M, (int)Wp, l.ff_p) * M * Wp * 4);
            act = max_of(act, M * l.ff_p * es);
        }
        for (int j = 0; j < l.n_mixers; j++) {
            const nc_stack_mixer& x = l.mix[j];
            switch (x.kind) {
                case NC_MIXER_LATENT_ATTENTION: {
                    const NcLatentGeom g = latent_geom(x, B, T, max_keys, max_keys - T);
                    if (expand(m->dtype, x, g)) {
                        kv = max_of(kv, (size_t)B * max_keys * x.heads * (x.dim_p + x.vdim_p) * es);
                    } else {
                        qlat = max_of(qlat, M * x.heads * (x.rank_p + x.rot_p) * es);
                        olat = max_of(olat, M * x.heads * x.rank_p * es);
                        att = max_of(att, nc_latent_partial_bytes(m->dtype, g));
                    }
                    break;
                }
                case NC_MIXER_RETENTION:
                    ret = max_of(ret, nc_retention_workspace_bytes(m->dtype, retention_geom(x, B, T, nullptr)));
                    if (x.gate == NC_GATE_JOINT_NORM_SIGMOID) raw = max_of(raw, M * x.heads * x.vdim_p * 4);
                    break;
                case NC_MIXER_WINDOW_ATTENTION:
                    att = max_of(att, nc_window_partial_bytes(m->dtype, window_geom(x, B, T, max_keys, max_keys - T)));
                    break;
                default:
                    ret = max_of(ret, nc_scan_workspace_bytes(scan_geom(x, B, T)));
                    u = max_of(u, M * x.inner_p * es);
                    x_parts = max_of(x_parts, (size_t)scan_x_splits(x, (int)M) * M * scan_x_cols(x) * 4);
                    if (T == 1) break;
                    dt = max_of(dt, M * x.inner_p * 4);
                    dtr = max_of(dtr, M * x.dt_rank_p * es), bc = max_of(bc, M * 2 * nc_scan_bc_cols(x.state_p) * 4);
            }
        }
        if (l.ff == NC_FF_EXPERTS) {
            const size_t p = M * l.top;
            pairs = max_of(pairs, p);
            tiles = max_of(tiles, expert_max_tiles(l, (int)M, expert_tile_rows(l, (int)M)));
            act = max_of(act, p * l.expert_ff_p * es);
            eout = max_of(eout, p * Wp * es);
        }
    }
    Carver c(base);
    Workspace w;
    w.x = (float*)c.take(M * Wp * 4);
    w.x0 = (float*)c.take(again ? M * Wp * 4 : 0);
    w.h = c.take(M * Wp * es);
    w.proj = c.take(proj);
    w.cat = c.take(M * m->max_k_out * es);
    w.router = (float*)c.take(router);
    w.h_last = c.take((size_t)n_logits * Wp * es);
    w.part_bytes = parts;
    w.parts = (float*)c.take(parts);
    w.q_lat = c.take(qlat);
    w.o_lat = c.take(olat);
    w.kv = c.take(kv);
    w.att_part_bytes = att;
    w.att_parts = c.take(att);
    w.ret = c.take(ret);
    w.act = c.take(act);
    w.e_out = c.take(eout);
    w.slot_w = (float*)c.take(pairs * 4);
    w.chosen = (int32_t*)c.take(pairs * 4);
    w.slot_of = (int32_t*)c.take(pairs * 4);
    w.perm = (int32_t*)c.take(pairs * 4);
    w.tiles = (int32_t*)c.take(tiles * NC_TILE_WORDS * 4);
    w.n_tiles = (int32_t*)c.take(4);
    w.raw = (float*)c.take(raw);
    w.u = c.take(u);
    w.dtr = c.take(dtr);
    w.bc = (float*)c.take(bc);
    w.dt = (float*)c.take(dt);
    w.x_parts = (float*)c.take(x_parts);
    w.total = (c.off + 255) & ~(size_t)255;
    return w;
}

const void* at(const void* p, int64_t elems, int dtype) { return (const uint8_t*)p + elems * (dtype ? 4 : 2); }
void* at(void* p, int64_t elems, int dtype) { return (uint8_t*)p + elems * (dtype ? 4 : 2); }

int run_linear(int dtype, const NcLinear& l, hipStream_t s) {
    return l.M <= NC_FEW_ROWS || l.K % 64 != 0 ? nc_launch_linear_few(dtype, l, s) : nc_launch_linear_tiled(dtype, l, s);
}

// A mixer reads its columns of the projected rows (`proj`, leading dimension ldp) and writes its columns of what the output matrix multiplies
// (`cat`, leading dimension ld_cat).
int run_latent_attention(int dt, const nc_stack_mixer& l, const NcLatentGeom& g, const Workspace& w, void* proj, int ldp, float eps, int rope_len,
                         const int32_t* seqlens, void* cache, void* cat, int ld_cat, hipStream_t s) {
    const int M = g.B * g.T, qd = l.dim_p + l.rot_p, rw = l.rank_p + l.rot_p, head_w = l.dim_p + l.vdim_p;
    const bool ex = expand(dt, l, g);
    TRY(nc_launch_latent_append(dt, g, proj, ldp, l.kv_norm_w, eps, l.rope, rope_len, seqlens, cache, ex ? nullptr : w.q_lat, s));
    if (ex) {
        const int keys = g.pos_max + g.T;
        NcLinear e = nc_linear(cache, rw, l.w_ukv, keys, l.heads * head_w, l.rank_p);
        e.batch = g.B, e.a_stride = (int64_t)g.Tmax * rw, e.w_stride = 0, e.out_stride = (int64_t)keys * l.heads * head_w;
        nc_linear_seg(e, e.N, NC_SEG_PLAIN, w.kv, l.heads * head_w);
        TRY(nc_launch_linear_tiled(dt, e, s));
        return nc_launch_latent_expanded(g, (const bf16_t*)proj, ldp, (const bf16_t*)w.kv, keys, (const bf16_t*)cache, seqlens, (bf16_t*)cat, ld_cat, s);
    }
    // unrotated queries into latent space, one product per head
    NcLinear q = nc_linear(proj, ldp, l.w_uk_t, M, l.rank_p, l.dim_p);
    q.batch = l.heads, q.a_stride = qd, q.w_stride = (int64_t)l.rank_p * l.dim_p, q.out_stride = rw;
    nc_linear_seg(q, q.N, NC_SEG_PLAIN, w.q_lat, l.heads * rw);
    TRY(run_linear(dt, q, s));
    TRY(nc_launch_latent_attention(dt, g, w.q_lat, cache, seqlens, w.o_lat, w.att_parts, w.att_part_bytes, s));
    // ... and the weighted latents out of it: the value rows of w_ukv sit behind the head's dim_p key rows
    NcLinear v = nc_linear(w.o_lat, l.heads * l.rank_p, at(l.w_ukv, (int64_t)l.dim_p * l.rank_p, dt), M, l.vdim_p, l.rank_p);
    v.batch = l.heads, v.a_stride = l.rank_p, v.w_stride = (int64_t)head_w * l.rank_p, v.out_stride = l.vdim_p;
    nc_linear_seg(v, v.N, NC_SEG_PLAIN, cat, ld_cat);
    return run_linear(dt, v, s);
}

int run_window_attention(int dt, const nc_stack_mixer& l, const NcWindowGeom& g, const Workspace& w, void* proj, int ldp, float eps, int rope_len,
                         const int32_t* seqlens, void* cache, void* cat, int ld_cat, hipStream_t s) {
    TRY(nc_launch_window_append(dt, g, proj, ldp, l.qkv_bias, l.q_norm_w, l.k_norm_w, eps, l.rope, rope_len, seqlens, cache, s));
    return nc_launch_window_attention(dt, g, proj, ldp, cache, l.sink, seqlens, cat, ld_cat, w.att_parts, w.att_part_bytes, s);
}

int run_retention(int dt, const nc_stack_mixer& l, const NcRetentionGeom& g, const Workspace& w, const void* proj, int ldp, float eps, int rope_len,
                  const int32_t* seqlens, const float* state_in, float* state_out, void* cat, int ld_cat, hipStream_t s) {
    TRY(nc_launch_retention(dt, g, proj, ldp, l.decay, l.rope, rope_len, seqlens, state_in, state_out, eps, cat, ld_cat, w.ret, s));
    if (!g.raw) return 0;
    const void* gate = at(proj, (int64_t)l.heads * (2 * l.dim_p + l.vdim_p), dt);
    return nc_launch_joint_gate(dt, g.raw, l.heads * l.vdim_p, l.heads * l.vdim, gate, ldp, l.out_norm_w, eps, l.out_scale, cat, ld_cat, g.B * g.T, s);
}

int run_selective_scan(int dt, const nc_stack_mixer& l, const NcScanGeom& g, const Workspace& w, const void* proj, int ldp, const int32_t* seqlens,
                       const float* state_in, float* state_out, void* cat, int ld_cat, hipStream_t s) {
    const int M = g.B * g.T, N = scan_x_cols(l), splits = scan_x_splits(l, M);
    TRY(nc_launch_scan_conv(dt, g, proj, ldp, l.conv_w, l.conv_b, seqlens, state_in, state_out, w.u, s));
    NcLinear x = nc_linear(w.u, l.inner_p, l.w_x, M, N, l.inner_p);
    if (M <= NC_FEW_ROWS) {
        if (splits > 1) x.partials = w.x_parts, x.splits = splits;
        else nc_linear_seg(x, N, NC_SEG_F32, w.x_parts, N);
    } else {                                       // every share is a product of its own
        x.K = l.inner_p / splits, x.batch = splits, x.a_stride = x.w_stride = x.K, x.out_stride = (int64_t)M * N;
        nc_linear_seg(x, N, NC_SEG_F32, w.x_parts, N);
    }
    TRY(run_linear(dt, x, s));
    const void* z = at(proj, l.inner_p, dt);
    if (g.T == 1) {
        const NcScanStep p{w.x_parts, splits, l.w_dt_t, l.dt_b, l.a_log2, l.skip, w.u, z, ldp, seqlens, state_in, state_out, cat, ld_cat};
        return nc_launch_scan_step(dt, g, p, s);
    }
    TRY(nc_launch_scan_join(dt, g, w.x_parts, splits, w.dtr, w.bc, s));
    NcLinear d = nc_linear(w.dtr, l.dt_rank_p, l.w_dt, M, l.inner_p, l.dt_rank_p);
    nc_linear_seg(d, d.N, NC_SEG_SOFTPLUS, w.dt, l.inner_p, 0.f, 0.f, l.dt_b);
    TRY(run_linear(dt, d, s));
    return nc_launch_scan(dt, g, w.u, w.dt, w.bc, l.a_log2, l.skip, z, ldp, seqlens, state_in, state_out, cat, ld_cat, w.ret, s);
}

// The mixers of one layer run, on the projected rows w.proj, into w.cat.
int run_mixers(const nc_stack_model* m, const nc_stack_cache* kv, const nc_stack_run& run, const Workspace& w, int B, int T, hipStream_t s) {
    const nc_stack_layer& l = m->layers[run.layer];
    const int dt = m->dtype;
    int col = 0, to = 0;
    for (int j = 0; j < l.n_mixers; j++) {
        const nc_stack_mixer& x = l.mix[j];
        const int slot = run.slot[j];
        void *proj = at(w.proj, col, dt), *cat = at(w.cat, to, dt);
        switch (x.kind) {
            case NC_MIXER_LATENT_ATTENTION:
                TRY(run_latent_attention(dt, x, latent_geom(x, B, T, kv->max_seq_len, kv->pos_max), w, proj, l.mix_cols, m->eps, m->rope_len, kv->cache_seqlens,
                                         kv->rows[slot], cat, l.k_out, s));
                break;
            case NC_MIXER_RETENTION:
                TRY(run_retention(dt, x, retention_geom(x, B, T, x.gate == NC_GATE_JOINT_NORM_SIGMOID ? w.raw : nullptr), w, proj, l.mix_cols, m->eps, m->rope_len,
                                  kv->cache_seqlens, kv->state_in[slot], kv->state_out[slot], cat, l.k_out, s));
                break;
            case NC_MIXER_WINDOW_ATTENTION:
                TRY(run_window_attention(dt, x, window_geom(x, B, T, kv->max_seq_len, kv->pos_max), w, proj, l.mix_cols, m->eps, m->rope_len, kv->cache_seqlens,
                                         kv->rows[slot], cat, l.k_out, s));
                break;
            default:
                TRY(run_selective_scan(dt, x, scan_geom(x, B, T), w, proj, l.mix_cols, kv->cache_seqlens, kv->state_in[slot], kv->state_out[slot], cat, l.k_out, s));
        }
        col += x.cols, to += x.out;
    }
    return 0;
}
// The columns of the input matrix that are the mixers' own.
void mixer_segs(const nc_stack_layer& l, NcLinear& in, const Workspace& w, int dt) {
    int col = 0;
    for (int j = 0; j < l.n_mixers; j++) {
        const nc_stack_mixer& x = l.mix[j];
        int from = col;
        if (x.silu_qkv) {
            const int qkv = x.heads * (2 * x.dim_p + x.vdim_p);
            nc_linear_seg(in, col + qkv, NC_SEG_SILU, at(w.proj, col, dt), l.mix_cols);
            from += qkv;
        }
        nc_linear_seg(in, col + x.cols, NC_SEG_PLAIN, at(w.proj, from, dt), l.mix_cols);
        col += x.cols;
    }
}

int run_experts(int dt, const nc_stack_layer& l, int M, int width_p, const Workspace& w, hipStream_t s) {
    NcRoute r{};
    r.logits = w.router, r.ld = l.router_cols, r.experts = l.experts, r.top = l.top;
    r.slot_w = w.slot_w, r.chosen = w.chosen, r.slot_of = w.slot_of, r.perm = w.perm, r.tiles = w.tiles, r.n_tiles = w.n_tiles;
    r.tile_rows = expert_tile_rows(l, M), r.max_tiles = expert_max_tiles(l, M, r.tile_rows);
    TRY(nc_launch_stack_route(r, M, s));
    const int pairs = M * l.top;
    auto grouped = [&](NcLinear& g) {
        g.tiles = w.tiles, g.n_tiles = w.n_tiles, g.max_tiles = r.max_tiles, g.tile_rows = r.tile_rows, g.w_stride = (int64_t)g.N * g.K;
        return r.tile_rows == NC_GROUP_TILE_FEW ? nc_launch_linear_few(dt, g, s, NC_CLS_EXPERTS) : nc_launch_linear_tiled(dt, g, s, NC_CLS_EXPERTS);
    };
    NcLinear up = nc_linear(w.h, width_p, l.w_e1, pairs, 2 * l.expert_ff_p, width_p);
    up.a_rows = w.perm, up.a_div = l.top;
    nc_linear_seg(up, up.N, NC_SEG_GLU, w.act, l.expert_ff_p, l.expert_limit);
    TRY(grouped(up));
    NcLinear down = nc_linear(w.act, l.expert_ff_p, l.w_e2, pairs, width_p, l.expert_ff_p);
    nc_linear_seg(down, down.N, NC_SEG_PLAIN, w.e_out, width_p);
    return grouped(down);
}

int check_mixer(const nc_stack_mixer& x, int i) {
    NC_CHECK_ARG(x.cols % 16 == 0 && x.out % 16 == 0 && (x.rope || x.rot_dims == 0), "stack: layer %d mixer columns", i);
    const bool scales = x.kind == NC_MIXER_WINDOW_ATTENTION || x.kind == NC_MIXER_SELECTIVE_SCAN || (x.kind == NC_MIXER_RETENTION && x.gate);
    NC_CHECK_ARG(scales || x.out_scale == 1.f, "stack: layer %d: a mixer of this kind does not scale its result", i);
    if (x.kind != NC_MIXER_SELECTIVE_SCAN) NC_CHECK_ARG(x.out == x.heads * x.vdim_p, "stack: layer %d output columns", i);
    switch (x.kind) {
        case NC_MIXER_LATENT_ATTENTION:
            NC_CHECK_ARG(x.kv_norm_w && x.w_uk_t && x.w_ukv, "stack: layer %d has no latent weights", i);
            NC_CHECK_ARG(x.dim_p % 32 == 0 && x.rot_p % 32 == 0 && x.vdim_p % 16 == 0 && x.rank_p % NC_STACK_PAD == 0 &&
                             x.cols == x.heads * (x.dim_p + x.rot_p) + x.rank_p + x.rot_p, "stack: layer %d latent sizes", i);
            return 0;
        case NC_MIXER_RETENTION:
            NC_CHECK_ARG(x.decay && (!x.gate || x.out_norm_w), "stack: layer %d has no retention weights", i);
            NC_CHECK_ARG(x.dim_p % 16 == 0 && x.vdim_p % 16 == 0 && x.cols == 2 * x.heads * (x.dim_p + x.vdim_p), "stack: layer %d retention sizes", i);
            return 0;
        case NC_MIXER_WINDOW_ATTENTION:
            NC_CHECK_ARG(x.qkv_bias && x.q_norm_w && x.k_norm_w && x.sink, "stack: layer %d has no window attention weights", i);
            NC_CHECK_ARG(x.kv_heads >= 1 && x.heads % x.kv_heads == 0 && x.dim_p % 32 == 0 && x.vdim_p % 16 == 0 &&
                             x.cols == (x.heads + x.kv_heads) * x.dim_p + x.kv_heads * x.vdim_p, "stack: layer %d window attention sizes", i);
            return 0;
        case NC_MIXER_SELECTIVE_SCAN:
            NC_CHECK_ARG(x.conv_w && x.conv_b && x.w_x && x.w_dt && x.w_dt_t && x.dt_b && x.a_log2 && x.skip, "stack: layer %d has no scan weights", i);
            NC_CHECK_ARG(x.inner_p % NC_STACK_PAD == 0 && x.dt_rank_p % NC_STACK_PAD == 0 && x.state_p % 4 == 0 && x.taps >= 1 && x.cols == 2 * x.inner_p &&
                             x.out == x.inner_p, "stack: layer %d scan sizes", i);
            return 0;
    }
    NC_FAIL(-1, "stack: layer %d mixer", i);
}

int check_layer(const nc_stack_layer& l, int i) {
    NC_CHECK_ARG(l.w_in && l.w_out && l.norm_w, "stack: layer %d has no weights", i);
    NC_CHECK_ARG(l.n_mixers >= 1 && l.n_mixers <= NC_STACK_MAX_MIXERS, "stack: layer %d has %d mixers", i, l.n_mixers);
    int cols = 0, out = 0, segs = 0;
    for (int j = 0; j < l.n_mixers; j++) {
        TRY(check_mixer(l.mix[j], i));
        cols += l.mix[j].cols, out += l.mix[j].out, segs += l.mix[j].silu_qkv ? 2 : 1;
    }
    const bool post = l.block == NC_BLOCK_POST_NORM;
    NC_CHECK_ARG(l.block == NC_BLOCK_PARALLEL || post, "stack: layer %d block", i);
    NC_CHECK_ARG(cols == l.mix_cols && l.router_cols % 16 == 0 && l.ff_cols % 16 == 0 && l.n_in == l.mix_cols + (post ? 0 : l.router_cols + l.ff_cols),
                 "stack: layer %d input columns", i);
    NC_CHECK_ARG(out == l.mix_out && l.k_out == l.mix_out + (post ? 0 : l.ff_p) && l.k_out % NC_STACK_PAD == 0 && l.ff_p % NC_STACK_PAD == 0,
                 "stack: layer %d output columns", i);
    NC_CHECK_ARG(segs + (l.router_cols > 0) + (!post && l.ff_cols > 0) <= 4, "stack: layer %d has too many parts", i);
    const bool dense = l.ff == NC_FF_DENSE_GELU || l.ff == NC_FF_DENSE_SWIGLU;
    if (post) NC_CHECK_ARG(l.ff == NC_FF_NONE || (dense && l.w_ff_in && l.w_ff_out && l.norm2_w && l.ff_p > 0), "stack: layer %d feed-forward", i);
    if (l.ff == NC_FF_EXPERTS)
        NC_CHECK_ARG(l.w_e1 && l.w_e2 && l.router_cols >= l.experts && l.top >= 1 && l.top <= l.experts && l.expert_ff_p % NC_STACK_PAD == 0 &&
                         l.ff_cols == 2 * l.ff_p, "stack: layer %d expert sizes", i);
    else
        NC_CHECK_ARG(l.router_cols == 0 && l.ff_cols == (l.ff == NC_FF_DENSE_SWIGLU ? 2 : 1) * l.ff_p && (dense || (l.ff == NC_FF_NONE && l.ff_p == 0)),
                     "stack: layer %d feed-forward sizes", i);
    return 0;
}
int ff_seg_kind(int ff) { return ff == NC_FF_EXPERTS ? NC_SEG_GLU : ff == NC_FF_DENSE_SWIGLU ? NC_SEG_SWIGLU : NC_SEG_GELU; }
// how the rows that enter a run's first linear come out of x
void entry_norm(const nc_stack_model* m, const nc_stack_run& run, int& norm, const float*& w) {
    const nc_stack_layer& l = m->layers[run.layer];
    norm = l.block == NC_BLOCK_POST_NORM ? NC_ROW_COPY : m->norm == NC_NORM_RMS ? NC_ROW_RMS_NORM : NC_ROW_LAYER_NORM;
    w = l.norm_w;
}
// sums = W rows, in fp32 for the row kernel: whole, or (few rows) in as many shares as fill the chip
int run_sums(int dt, const void* a, const void* w, int M, int N, int K, float* parts, NcRowAdd& add, hipStream_t s) {
    NcLinear l = nc_linear(a, K, w, M, N, K);
    const int splits = M <= NC_FEW_ROWS ? nc_linear_few_splits(M, N, K) : 1;
    if (splits > 1) l.partials = parts, l.splits = splits;
    else nc_linear_seg(l, N, NC_SEG_F32, parts, N);
    add.partials = parts, add.splits = splits;
    return run_linear(dt, l, s);
}
}  // namespace

extern "C" int nc_stack_abi_version(void) { return 2; }

extern "C" size_t nc_stack_workspace_bytes(const nc_stack_model* m, int B, int T, int n_logits, int max_keys) {
    if (!m || B <= 0 || T <= 0 || max_keys < T) return 0;
    return carve(m, B, T, n_logits, max_keys, nullptr).total;
}

extern "C" int nc_stack_forward(const nc_stack_model* m, const nc_stack_cache* kv, const int64_t* idx, int B, int T, const int32_t* logit_rows,
                                int n_logits, float* logits_out, void* workspace, size_t workspace_bytes, float* taps, nc_stream_t stream) {
    hipStream_t s = (hipStream_t)stream;
    NC_CHECK_ARG(m && kv && idx && workspace && (n_logits == 0 || logits_out), "stack_forward: null pointer");
    NC_CHECK_ARG(B > 0 && T > 0 && kv->batch == B && kv->cache_seqlens, "stack_forward: batch %d of a cache of %d rows", B, kv->batch);
    NC_CHECK_ARG(kv->pos_max >= 0 && kv->pos_max + T <= kv->max_seq_len, "stack_forward: a cache of %d tokens cannot take %d + %d", kv->max_seq_len, kv->pos_max, T);
    NC_CHECK_ARG(kv->pos_max + T <= m->rope_len, "stack_forward: position %d past the rotary tables", kv->pos_max + T);
    NC_CHECK_ARG(m->width_p % NC_STACK_PAD == 0 && m->n_runs >= 1, "stack_forward: width %d, %d runs", m->width_p, m->n_runs);
    NC_CHECK_ARG(logit_rows || n_logits == 0 || n_logits == B * T, "stack_forward: without a selection all rows have logits");
    NC_CHECK_ARG(!kv->advance || (!logit_rows && n_logits > 0), "stack_forward: the positions are advanced by the pass over all rows");
    NC_CHECK_ARG(((uintptr_t)workspace & 255) == 0, "stack_forward: workspace must be 256-byte aligned");
    for (int i = 0; i < m->n_layers; i++) TRY(check_layer(m->layers[i], i));
    const int M = B * T, Wp = m->width_p, dt = m->dtype;
    const int keys = kv->pos_max + T;
    // the caller sized the workspace for its own bound on the keys; what this call needs is never more than that
    const Workspace w = carve(m, B, T, n_logits, keys, workspace);
    NC_CHECK_ARG(workspace_bytes >= w.total, "stack_forward: workspace of %zu bytes needed, %zu given", w.total, workspace_bytes);
    bool again = false;
    for (int i = 0; i < m->n_runs; i++) {
        const nc_stack_run& r = m->runs[i];
        NC_CHECK_ARG(r.layer >= 0 && r.layer < m->n_layers && (r.step < 0 || m->steps), "stack_forward: run %d", i);
        again |= r.add_embedding != 0;
    }
    const int final_norm = m->norm == NC_NORM_RMS ? NC_ROW_RMS_NORM : NC_ROW_LAYER_NORM;
    int norm;
    const float* norm_w;
    entry_norm(m, m->runs[0], norm, norm_w);
    TRY(nc_launch_stack_embed(dt, idx, m->embed, m->embed_scale, m->runs[0].step >= 0 ? m->steps + (int64_t)m->runs[0].step * Wp : nullptr, m->vocab, w.x,
                              again ? w.x0 : nullptr, norm, norm_w, m->eps, w.h, M, m->width, Wp, s));
    for (int i = 0; i < m->n_runs; i++) {
        const nc_stack_run& run = m->runs[i];
        const nc_stack_layer& l = m->layers[run.layer];
        const bool post = l.block == NC_BLOCK_POST_NORM;
        NcLinear in = nc_linear(w.h, Wp, l.w_in, M, l.n_in, Wp);
        mixer_segs(l, in, w, dt);
        if (l.router_cols) nc_linear_seg(in, l.mix_cols + l.router_cols, NC_SEG_F32, w.router, l.router_cols);
        if (!post && l.ff_cols) nc_linear_seg(in, l.n_in, ff_seg_kind(l.ff), at(w.cat, l.mix_out, dt), l.k_out, l.ff_limit);
        TRY(run_linear(dt, in, s));
        TRY(run_mixers(m, kv, run, w, B, T, s));

        NcRowAdd add{};
        add.x = w.x, add.tokens_per_row = T;
        if (post) {
            TRY(run_sums(dt, w.cat, l.w_out, M, Wp, l.k_out, w.parts, add, s));
            add.post_norm_w = l.norm_w;
            if (l.ff) {
                add.norm = NC_ROW_COPY, add.h = w.h;
                TRY(nc_launch_stack_row_add(dt, add, m->eps, M, M, m->width, Wp, s));
                NcLinear up = nc_linear(w.h, Wp, l.w_ff_in, M, l.ff_cols, Wp);
                nc_linear_seg(up, l.ff_cols, ff_seg_kind(l.ff), w.act, l.ff_p);
                TRY(run_linear(dt, up, s));
                TRY(run_sums(dt, w.act, l.w_ff_out, M, Wp, l.ff_p, w.parts, add, s));
                add.post_norm_w = l.norm2_w, add.h = nullptr;
            }
        } else {
            if (l.ff == NC_FF_EXPERTS) TRY(run_experts(dt, l, M, Wp, w, s));
            NcLinear out = nc_linear(w.cat, l.k_out, l.w_out, M, Wp, l.k_out);
            const int splits = M <= NC_FEW_ROWS ? nc_linear_few_splits(M, Wp, l.k_out) : 1;
            if (splits > 1) out.partials = w.parts, out.splits = splits, add.partials = w.parts, add.splits = splits;
            else nc_linear_seg(out, Wp, NC_SEG_RESIDUAL, w.x, Wp);
            TRY(run_linear(dt, out, s));
            if (l.ff == NC_FF_EXPERTS) add.expert_out = w.e_out, add.slot_of = w.slot_of, add.slot_w = w.slot_w, add.top = l.top;
        }
        if (taps) add.tap = taps + (int64_t)i * M * Wp;
        if (i + 1 < m->n_runs) {
            const nc_stack_run& next = m->runs[i + 1];
            add.x0 = next.add_embedding ? w.x0 : nullptr;
            add.step = next.step >= 0 ? m->steps + (int64_t)next.step * Wp : nullptr;
            entry_norm(m, next, add.norm, add.norm_w);
            add.h = w.h;
            TRY(nc_launch_stack_row_add(dt, add, m->eps, M, M, m->width, Wp, s));
            continue;
        }
        if (taps) {                       // all rows, then the selection
            TRY(nc_launch_stack_row_add(dt, add, m->eps, M, M, m->width, Wp, s));
            add = NcRowAdd{};
            add.x = w.x, add.tokens_per_row = T;
        }
        if (n_logits == 0) return 0;
        add.norm = final_norm, add.norm_w = m->final_norm_w, add.h = w.h_last, add.rows = logit_rows;
        if (kv->advance) add.bump = kv->cache_seqlens, add.bump_by = kv->advance;
        TRY(nc_launch_stack_row_add(dt, add, m->eps, M, n_logits, m->width, Wp, s));
        NcLinear head = nc_linear(w.h_last, Wp, m->head, n_logits, m->vocab, Wp);
        nc_linear_seg(head, m->vocab, NC_SEG_LOGITS, logits_out, m->vocab, m->logit_scale, m->logit_softcap);
        TRY(run_linear(dt, head, s));
    }
    return 0;
}

extern "C" int nc_stack_linear(int dtype, const void* a, int64_t lda, const void* w, void* out, int ldc, int M, int N, int K, int kind, float limit,
                               int kernel, nc_stream_t stream) {
    NC_CHECK_ARG(out && ((kind >= NC_SEG_PLAIN && kind <= NC_SEG_F32) || kind == NC_SEG_SILU || kind == NC_SEG_SWIGLU) && N % 16 == 0 && kernel >= 0 && kernel <= 4, "stack_linear: kind %d, N %d", kind, N);
    NcLinear l = nc_linear(a, lda, w, M, N, K);
    nc_linear_seg(l, N, kind, out, ldc, limit);
    if (kernel == 0) return run_linear(dtype, l, (hipStream_t)stream);
    if (kernel == 1) return nc_launch_linear_few(dtype, l, (hipStream_t)stream);
    return nc_launch_linear_tiled(dtype, l, (hipStream_t)stream, NC_CLS_LINEAR, kernel - 2);
}

extern "C" int nc_stack_cache_copy(const void* src, void* dst, int src_rows, int dst_rows, int64_t src_row_bytes, int64_t dst_row_bytes, int64_t n_bytes,
                                   nc_stream_t stream) {
    return nc_launch_stack_cache_copy(src, dst, src_rows, dst_rows, src_row_bytes, dst_row_bytes, n_bytes, (hipStream_t)stream);
}
