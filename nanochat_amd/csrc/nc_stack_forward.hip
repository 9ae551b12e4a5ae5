// Host-side sequencing of one forward of the layer stack on a stream (include/nanochat_amd_stack.h): one call enqueues every kernel of
// the step; no host synchronisation, no allocation.
//
// Per layer run, h = the normed rows:
//   linear   [projections | router logits | first feed-forward matrix] . h    the activation of the feed-forward in the epilogue
//   mixer    latent attention or retention  -> its part of `cat`; the feed-forward's part is there already
//   experts  route (softmax, choice, expert order), gate and up with their activation, down: one row per (token, choice)
//   linear   w_out . cat, added to the residual stream: in its epilogue, or (few rows) as partial sums by the row kernel
//   row add  x += partial sums + weighted expert rows (+ embedding output + step vector at the start of a pass), layer norm -> h
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
    float *x, *x0, *router, *parts;
    void *h, *proj, *cat, *h_last, *q_lat, *o_lat, *kv, *att_parts, *ret, *act, *e_out;
    float* slot_w;
    int32_t *chosen, *slot_of, *perm, *tiles, *n_tiles;
    size_t att_part_bytes, part_bytes, total;
};

NcLatentGeom latent_geom(const nc_stack_layer& l, int B, int T, int Tmax, int pos_max) {
    return NcLatentGeom{l.heads, l.dim_p, l.rot_p, l.rot_dims, l.rank, l.rank_p, l.vdim_p, l.score_scale, B, T, Tmax, pos_max};
}
NcRetentionGeom retention_geom(const nc_stack_layer& l, int B, int T) {
    return NcRetentionGeom{l.heads, l.dim, l.dim_p, l.vdim, l.vdim_p, l.rot_dims, l.score_scale, B, T};
}
// Expanding keys and values costs rank (dim + vdim) per key and head; after that a (query, key) pair costs dim + rot + vdim and only the
// visible half of the new pairs is visited, against 2 rank + rot in latent space.
bool expand(int dtype, const nc_stack_layer& l, const NcLatentGeom& g) {
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
    size_t proj = 0, router = 0, parts = 0, qlat = 0, olat = 0, kv = 0, att = 0, ret = 0, act = 0, eout = 0, pairs = 0, tiles = 0;
    bool again = false;
    for (int i = 0; i < m->n_runs; i++) again |= m->runs[i].add_embedding != 0;
    for (int i = 0; i < m->n_layers; i++) {
        const nc_stack_layer& l = m->layers[i];
        proj = max_of(proj, M * l.mix_cols * es);
        router = max_of(router, M * l.router_cols * 4);
        if (M <= NC_FEW_ROWS) parts = max_of(parts, (size_t)nc_linear_few_splits((int)M, (int)Wp, l.k_out) * M * Wp * 4);
        if (l.mixer == NC_MIXER_LATENT_ATTENTION) {
            const NcLatentGeom g = latent_geom(l, B, T, max_keys, max_keys - T);
            if (expand(m->dtype, l, g)) {
                kv = max_of(kv, (size_t)B * max_keys * l.heads * (l.dim_p + l.vdim_p) * es);
            } else {
                qlat = max_of(qlat, M * l.heads * (l.rank_p + l.rot_p) * es);
                olat = max_of(olat, M * l.heads * l.rank_p * es);
                att = max_of(att, nc_latent_partial_bytes(m->dtype, g));
            }
        } else {
            ret = max_of(ret, nc_retention_workspace_bytes(m->dtype, retention_geom(l, B, T)));
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
    w.total = (c.off + 255) & ~(size_t)255;
    return w;
}

const void* at(const void* p, int64_t elems, int dtype) { return (const uint8_t*)p + elems * (dtype ? 4 : 2); }
void* at(void* p, int64_t elems, int dtype) { return (uint8_t*)p + elems * (dtype ? 4 : 2); }

int run_linear(int dtype, const NcLinear& l, hipStream_t s) {
    return l.M <= NC_FEW_ROWS || l.K % 64 != 0 ? nc_launch_linear_few(dtype, l, s) : nc_launch_linear_tiled(dtype, l, s);
}

int run_latent_attention(int dt, const nc_stack_layer& l, const NcLatentGeom& g, const Workspace& w, const float* kv_norm_w, float eps, const float* rope,
                         int rope_len, const int32_t* seqlens, void* cache, int ld_cat, hipStream_t s) {
    const int M = g.B * g.T, qd = l.dim_p + l.rot_p, rw = l.rank_p + l.rot_p, head_w = l.dim_p + l.vdim_p;
    const bool ex = expand(dt, l, g);
    TRY(nc_launch_latent_append(dt, g, w.proj, l.mix_cols, kv_norm_w, eps, rope, rope_len, seqlens, cache, ex ? nullptr : w.q_lat, s));
    if (ex) {
        const int keys = g.pos_max + g.T;
        NcLinear e = nc_linear(cache, rw, l.w_ukv, keys, l.heads * head_w, l.rank_p);
        e.batch = g.B, e.a_stride = (int64_t)g.Tmax * rw, e.w_stride = 0, e.out_stride = (int64_t)keys * l.heads * head_w;
        nc_linear_seg(e, e.N, NC_SEG_PLAIN, w.kv, l.heads * head_w);
        TRY(nc_launch_linear_tiled(dt, e, s));
        return nc_launch_latent_expanded(g, (const bf16_t*)w.proj, l.mix_cols, (const bf16_t*)w.kv, keys, (const bf16_t*)cache, seqlens, (bf16_t*)w.cat, ld_cat, s);
    }
    // unrotated queries into latent space, one product per head
    NcLinear q = nc_linear(w.proj, l.mix_cols, l.w_uk_t, M, l.rank_p, l.dim_p);
    q.batch = l.heads, q.a_stride = qd, q.w_stride = (int64_t)l.rank_p * l.dim_p, q.out_stride = rw;
    nc_linear_seg(q, q.N, NC_SEG_PLAIN, w.q_lat, l.heads * rw);
    TRY(run_linear(dt, q, s));
    TRY(nc_launch_latent_attention(dt, g, w.q_lat, cache, seqlens, w.o_lat, w.att_parts, w.att_part_bytes, s));
    // ... and the weighted latents out of it: the value rows of w_ukv sit behind the head's dim_p key rows
    NcLinear v = nc_linear(w.o_lat, l.heads * l.rank_p, at(l.w_ukv, (int64_t)l.dim_p * l.rank_p, dt), M, l.vdim_p, l.rank_p);
    v.batch = l.heads, v.a_stride = l.rank_p, v.w_stride = (int64_t)head_w * l.rank_p, v.out_stride = l.vdim_p;
    nc_linear_seg(v, v.N, NC_SEG_PLAIN, w.cat, ld_cat);
    return run_linear(dt, v, s);
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

int check_layer(const nc_stack_layer& l, int width_p, int i) {
    NC_CHECK_ARG(l.w_in && l.w_out && l.norm_w && l.rope, "stack: layer %d has no weights", i);
    NC_CHECK_ARG(l.mix_cols % 16 == 0 && l.router_cols % 16 == 0 && l.ff_cols % 16 == 0 && l.n_in == l.mix_cols + l.router_cols + l.ff_cols,
                 "stack: layer %d input columns", i);
    NC_CHECK_ARG(l.mix_out == l.heads * l.vdim_p && l.k_out == l.mix_out + l.ff_p && l.k_out % NC_STACK_PAD == 0 && l.ff_p % NC_STACK_PAD == 0,
                 "stack: layer %d output columns", i);
    if (l.mixer == NC_MIXER_LATENT_ATTENTION) {
        NC_CHECK_ARG(l.kv_norm_w && l.w_uk_t && l.w_ukv, "stack: layer %d has no latent weights", i);
        NC_CHECK_ARG(l.dim_p % 32 == 0 && l.rot_p % 32 == 0 && l.vdim_p % 16 == 0 && l.rank_p % NC_STACK_PAD == 0 &&
                         l.mix_cols == l.heads * (l.dim_p + l.rot_p) + l.rank_p + l.rot_p, "stack: layer %d latent sizes", i);
    } else {
        NC_CHECK_ARG(l.mixer == NC_MIXER_RETENTION && l.decay, "stack: layer %d mixer", i);
        NC_CHECK_ARG(l.dim_p % 16 == 0 && l.vdim_p % 16 == 0 && l.mix_cols == 2 * l.heads * (l.dim_p + l.vdim_p), "stack: layer %d retention sizes", i);
    }
    if (l.ff == NC_FF_EXPERTS)
        NC_CHECK_ARG(l.w_e1 && l.w_e2 && l.router_cols >= l.experts && l.top >= 1 && l.top <= l.experts && l.expert_ff_p % NC_STACK_PAD == 0 &&
                         l.ff_cols == 2 * l.ff_p, "stack: layer %d expert sizes", i);
    else
        NC_CHECK_ARG(l.router_cols == 0 && l.ff_cols == l.ff_p && (l.ff == NC_FF_DENSE_GELU || (l.ff == NC_FF_NONE && l.ff_p == 0)), "stack: layer %d feed-forward sizes", i);
    (void)width_p;
    return 0;
}
}  // namespace

extern "C" int nc_stack_abi_version(void) { return 1; }

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
    for (int i = 0; i < m->n_layers; i++) TRY(check_layer(m->layers[i], m->width_p, i));
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
    const int32_t* pos = kv->cache_seqlens;

    TRY(nc_launch_stack_embed(dt, idx, m->embed, m->embed_scale, m->runs[0].step >= 0 ? m->steps + (int64_t)m->runs[0].step * Wp : nullptr, m->vocab, w.x,
                              again ? w.x0 : nullptr, m->layers[m->runs[0].layer].norm_w, m->eps, w.h, M, m->width, Wp, s));
    for (int i = 0; i < m->n_runs; i++) {
        const nc_stack_run& run = m->runs[i];
        const nc_stack_layer& l = m->layers[run.layer];
        NcLinear in = nc_linear(w.h, Wp, l.w_in, M, l.n_in, Wp);
        nc_linear_seg(in, l.mix_cols, NC_SEG_PLAIN, w.proj, l.mix_cols);
        if (l.router_cols) nc_linear_seg(in, l.mix_cols + l.router_cols, NC_SEG_F32, w.router, l.router_cols);
        if (l.ff_cols)
            nc_linear_seg(in, l.n_in, l.ff == NC_FF_EXPERTS ? NC_SEG_GLU : NC_SEG_GELU, at(w.cat, l.mix_out, dt), l.k_out, l.ff_limit);
        TRY(run_linear(dt, in, s));

        if (l.mixer == NC_MIXER_LATENT_ATTENTION)
            TRY(run_latent_attention(dt, l, latent_geom(l, B, T, kv->max_seq_len, kv->pos_max), w, l.kv_norm_w, m->eps, l.rope, m->rope_len, pos,
                                     kv->latents[run.slot], l.k_out, s));
        else
            TRY(nc_launch_retention(dt, retention_geom(l, B, T), w.proj, l.mix_cols, l.decay, l.rope, m->rope_len, pos, kv->state_in[run.slot],
                                    kv->state_out[run.slot], m->eps, w.cat, l.k_out, w.ret, s));
        if (l.ff == NC_FF_EXPERTS) TRY(run_experts(dt, l, M, Wp, w, s));

        NcRowAdd add{};
        add.x = w.x, add.tokens_per_row = T;
        NcLinear out = nc_linear(w.cat, l.k_out, l.w_out, M, Wp, l.k_out);
        const int splits = M <= NC_FEW_ROWS ? nc_linear_few_splits(M, Wp, l.k_out) : 1;
        if (splits > 1) out.partials = w.parts, out.splits = splits, add.partials = w.parts, add.splits = splits;
        else nc_linear_seg(out, Wp, NC_SEG_RESIDUAL, w.x, Wp);
        TRY(run_linear(dt, out, s));
        if (l.ff == NC_FF_EXPERTS) add.expert_out = w.e_out, add.slot_of = w.slot_of, add.slot_w = w.slot_w, add.top = l.top;
        if (taps) add.tap = taps + (int64_t)i * M * Wp;
        if (i + 1 < m->n_runs) {
            const nc_stack_run& next = m->runs[i + 1];
            add.x0 = next.add_embedding ? w.x0 : nullptr;
            add.step = next.step >= 0 ? m->steps + (int64_t)next.step * Wp : nullptr;
            add.norm_w = m->layers[next.layer].norm_w, add.h = w.h;
            TRY(nc_launch_stack_row_add(dt, add, m->eps, M, M, m->width, Wp, s));
            continue;
        }
        if (taps) {                       // all rows, then the selection
            TRY(nc_launch_stack_row_add(dt, add, m->eps, M, M, m->width, Wp, s));
            add = NcRowAdd{};
            add.x = w.x, add.tokens_per_row = T;
        }
        if (n_logits == 0) return 0;
        add.norm_w = m->final_norm_w, add.h = w.h_last, add.rows = logit_rows;
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
    NC_CHECK_ARG(out && kind >= 0 && kind <= 3 && N % 16 == 0 && kernel >= 0 && kernel <= 4, "stack_linear: kind %d, N %d", kind, N);
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
