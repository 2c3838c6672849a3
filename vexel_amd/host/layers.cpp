// Mixer programs: the executor of models whose layers are described one by one (model.h: MixLayer), over mixed batches.
//
// A step is a set of sequences with any number of new tokens each. Its rows run through every layer together:
//   norm | input projection (K and V leave for the paged pool on the way) | attention and / or convolution + scan | output
//   projection | norm, residual, norm | gate|up with SiLU | down | norm, residual, and the next layer's norm
// or, with a mixer and experts that read the same normed input,
//   norm | input projection with the router | routing | heads to their places, attention, or decaying states with their norm and
//   gate | output projection | experts' gate|up | down | residual with all of them, and the next layer's norm
// or, with the norm behind the residual sum and latent attention,
//   input projection (queries turned on the way) | norms, latents to the paged pool | queries into the latents' space |
//   attention | results out of it | output projection | residual, norm | up | activation | down | residual, norm, average
// or, with a layer norm on what a sublayer adds,
//   input projection | heads to their places, or gates | attention, or states and their norm | output projection | norm, residual |
//   up | down, or router | routing | experts' up | down | norm, residual
// The block tables, the pool's bookkeeping and the sequence slots are the runtime's own; recurrent state lies in one slot
// per sequence (the row of its block table), and a sequence at position 0 starts from nothing whatever the slot holds.
#include <math.h>
#include <string.h>

#include <set>
#include <type_traits>

#include "model.h"

namespace vh {

namespace {

int pad_to(int n, int m) { return (n + m - 1) / m * m; }
size_t esize(const MixModel &x) { return x.act == VX_ACT_F32 ? 4 : 2; }

int by_heads_ldq(const AttnMixer &t) { return pad_to(t.heads * t.maps * t.k_dim, 8); }

struct Widths {
    int width_pad = 0, in = 0, out = 0, xc = 0, dtr = 0, bc = 0, dt = 0, act = 0;
    int qc = 0, qa = 0, rot = 0;
    int o = 0, e_act = 0, e_out = 0, top = 0, places = 0, experts = 0;  // top, places: of a row
};

Widths widths(const vh_model *m) {
    Widths w;
    w.width_pad = pad_to(m->cfg.hidden, 64);
    for (const MixLayer &l : m->mix->layers) {
        w.in = std::max(w.in, l.has_latent                    ? l.latent.heads * l.latent.head_cols
                              : l.has_decay                     ? l.decay.split
                              : l.has_forget                    ? l.forget.heads * (l.forget.dim_pad + l.forget.v_pad)
                              : l.has_attn && l.attn.by_heads ? by_heads_ldq(l.attn)
                                                                : l.in.n);
        w.out = std::max(w.out, l.out.k);
        w.act = std::max(w.act, l.ff_pad);
        if (l.has_scan) {
            w.xc = std::max(w.xc, l.scan.x.k);
            w.dtr = std::max(w.dtr, l.scan.dt_pad);
            w.bc = std::max(w.bc, 2 * l.scan.pad);
            w.dt = std::max(w.dt, l.scan.dt.n);
        }
        if (l.has_latent) {
            w.qc = std::max(w.qc, l.latent.q_up.k);
            w.qa = std::max(w.qa, l.latent.heads * l.latent.rank_pad);
        }
    }
    for (const MixLayer &l : m->mix->layers) {
        if (l.has_decay) w.o = std::max(w.o, l.decay.heads * l.decay.v_pad);
        if (l.has_forget) w.o = std::max(w.o, l.forget.heads * l.forget.v_pad);
        if (l.has_experts) {
            const ExpertMlp &e = l.moe;
            w.e_act = std::max({w.e_act, e.ff_pad, e.shared_pad});
            w.e_out = std::max(w.e_out, e.down.n);
            w.top = std::max(w.top, e.top), w.places = std::max(w.places, e.top + (e.shared ? 1 : 0));
            w.experts = std::max(w.experts, e.experts);
        }
    }
    for (const Rotation &r : m->mix->rotations) w.rot += 2 * (int)r.freqs.size();
    return w;
}

// bytes of the up projection's output in front of vx_poly_norm, which may come as float32 slices
size_t up_bytes(const vh_model *m, int rows, bool up_to) {
    size_t most = 1;
    for (const MixLayer &l : m->mix->layers) {
        if (!l.poly) continue;
        for (int r = up_to ? 1 : rows; r <= rows; r++) {
            const size_t cut = vx_linear_slices(m->be, l.gate_up.n, l.gate_up.k, r);
            most = std::max(most, (size_t)r * l.ff_pad * (cut > 1 ? cut * 4 : esize(*m->mix)));
        }
    }
    return most;
}

// floats of sliced sublayer outputs, and of latent projections, that a step of up to `rows` rows may need
size_t slice_floats(const vh_model *m, int rows, bool up_to) {
    size_t most = 1;
    const auto sliced = [&](const Linear &w, int cols) {
        if (!w.w) return;
        for (int r = up_to ? 1 : rows; r <= rows; r++) most = std::max(most, (size_t)r * vx_linear_slices(m->be, w.n, w.k, r) * cols);
    };
    const int cols = pad_to(m->cfg.hidden, 16);
    for (const MixLayer &l : m->mix->layers) {
        sliced(l.out, cols);
        sliced(l.down, cols);
        if (l.has_attn && l.attn.by_heads) sliced(l.in, l.in.n);
        if (l.has_experts) sliced(l.moe.router, l.moe.router.n);
        if (l.has_forget) most = std::max(most, (size_t)rows * l.forget.heads * l.forget.dim_pad);
        if (l.has_decay) most = std::max(most, (size_t)rows * (l.in.n - l.decay.split));
        if (!l.has_latent) continue;
        if (l.latent.q_rank > 0)
            sliced(l.in, l.in.n);
        else
            most = std::max(most, (size_t)rows * l.latent.kv_cols);
    }
    return most;
}

template <class A>
int alloc_acts(vh_model *m, int rows, bool up_to, A &&alloc, MixActs *a) {
    const Widths w = widths(m);
    const size_t es = esize(*m->mix), R = rows;
    bool loop = false;
    for (const LayerRun &r : m->mix->runs) loop = loop || r.add_embedding;
    auto get = [&](auto **p, size_t bytes) {
        *p = (std::remove_reference_t<decltype(*p)>)alloc(bytes ? bytes : 16);
        return *p != nullptr;
    };
    a->rows = rows;
    const bool ok = get(&a->x, R * m->cfg.hidden * 4) && get(&a->h, R * w.width_pad * es) && get(&a->proj, R * w.in * es) &&
                    get(&a->cat, R * w.out * es) && get(&a->xc, R * w.xc * es) && get(&a->dtr, R * w.dtr * es) &&
                    get(&a->bc, R * w.bc * 4) && get(&a->dt, R * w.dt * 4) && get(&a->act, R * w.act * es) &&
                    get(&a->y, slice_floats(m, rows, up_to) * 4) && (!loop || get(&a->emb, R * m->cfg.hidden * 4)) &&
                    get(&a->qc, R * w.qc * es) && get(&a->qa, R * w.qa * es) && get(&a->lo, R * w.qa * es) && get(&a->z, up_bytes(m, rows, up_to)) &&
                    get(&a->rot, R * w.rot * 4) && get(&a->o, R * w.o * 4) && get(&a->e_act, R * w.places * w.e_act * es) &&
                    get(&a->e_out, R * w.places * w.e_out * es) && get(&a->e_weights, R * w.top * 4) && get(&a->e_places, R * w.top * 4) &&
                    get(&a->e_order, R * w.places * 4) &&
                    get(&a->e_tiles, w.top > 0 ? (4 + 4 * (size_t)vx_route_max_tiles(rows, w.experts, w.top, 1, 64)) * 4 : 0) &&
                    (!m->mix->post_norm || get(&a->hist, R * m->cfg.hidden * (m->mix->runs.size() + 1) * 4));
    return ok ? (int)VH_OK : fail("activations of %d rows: %s", rows, vx_last_error());
}

}  // namespace

int mix_finish(vh_model *m) {
    MixModel &x = *m->mix;
    const vh_config &c = m->cfg;
    const size_t es = esize(x);
    auto zeroed = [&](size_t bytes) {
        bytes = (bytes + 15) / 16 * 16;
        void *p = vx_alloc_permanent(m->be, bytes ? bytes : 16);
        if (p && vx_fill_zero(m->be, p, bytes ? bytes : 16) != VX_OK) {
            vx_free(m->be, p);
            p = nullptr;
        }
        return p;
    };
    for (LayerRun &r : x.runs) {
        const MixLayer &l = x.layers[r.layer];
        m->kv.push_back(nullptr);
        if (l.has_attn && l.attn.kv_from < 0) {
            // (what a kernel may read beyond a sequence's tokens is a finite number from the start)
            r.kv = zeroed(vx_kv_block_elems2(c.block_size, l.attn.kv_heads * l.attn.maps, l.attn.k_dim, l.attn.kv_heads, l.attn.v_dim) * c.pool_blocks * es);
            if (!r.kv) return fail("KV pool: %s", vx_last_error());
            m->kv.back() = r.kv;
        }
        if (l.has_latent && l.latent.kv_from < 0) {
            r.kv = zeroed((size_t)c.block_size * c.pool_blocks * l.latent.row * es);
            if (!r.kv) return fail("latent pool: %s", vx_last_error());
            m->kv.back() = r.kv;
        }
        if (l.has_latent && l.latent.kv_from >= 0)  // (every layer runs once in a model that shares pools)
            r.kv = x.runs[l.latent.kv_from].kv;
        if (l.has_attn && l.attn.kv_from >= 0) r.kv = x.runs[l.attn.kv_from].kv;
        if (l.has_scan) {
            r.state = (float *)zeroed((size_t)c.max_seqs * l.scan.channels * l.scan.pad * 4);
            if (!r.state) return fail("scan state: %s", vx_last_error());
            m->adopted.push_back(r.state);
            r.conv = zeroed((size_t)c.max_seqs * (l.scan.taps - 1) * l.scan.channels * es);
            if (!r.conv) return fail("convolution state: %s", vx_last_error());
            m->adopted.push_back(r.conv);
        }
    }
    for (LayerRun &r : x.runs) {
        const MixLayer &l = x.layers[r.layer];
        if (!l.has_decay && !l.has_forget) continue;
        const size_t per = l.has_decay ? (size_t)l.decay.heads * l.decay.dim_pad * l.decay.v_pad : (size_t)l.forget.heads * l.forget.dim_pad * l.forget.v_pad;
        r.state = (float *)zeroed(c.max_seqs * per * 4);
        if (!r.state) return fail("states: %s", vx_last_error());
        m->adopted.push_back(r.state);
    }
    if (x.pairs) {
        x.token_pool = (int32_t *)zeroed((size_t)c.block_size * c.pool_blocks * 4);
        if (!x.token_pool) return fail("token pool: %s", vx_last_error());
        m->adopted.push_back(x.token_pool);
    }
    for (Rotation &r : x.rotations) {
        void *p = vx_alloc_permanent(m->be, (r.freqs.size() * 8 + 15) / 16 * 16);
        if (!p) return fail("device memory: %s", vx_last_error());
        m->adopted.push_back(p);
        VXC(vx_to_device(m->be, p, r.freqs.data(), r.freqs.size() * 8));
        r.d_freqs = (const double *)p;
    }
    VHC(init_common(m));
    VHC(alloc_acts(m, c.max_batch, true, [&](size_t n) {
        void *p = vx_alloc_permanent(m->be, n);
        if (p) m->adopted.push_back(p);
        return p;
    }, &x.perm));
    VXC(vx_sync(m->be));
    return VH_OK;
}

namespace {

vx_linear_out plain(void *out, int out_f32, int ldo, int cols, int slices) {
    vx_linear_out o;
    memset(&o, 0, sizeof o);
    o.kind = VX_LIN_PLAIN;
    o.out = out, o.out_f32 = out_f32, o.ldo = ldo, o.cols = cols, o.slices = slices;
    return o;
}

void *at(void *p, size_t elems, size_t es) { return (char *)p + elems * es; }

// a rotation's angles of the step's rows
const float *rot_table(const MixModel &x, const MixActs &a, int rows, int rotation) {
    if (rotation < 0) return nullptr;
    size_t before = 0;
    for (int i = 0; i < rotation; i++) before += x.rotations[i].freqs.size();
    return a.rot + before * 2 * rows;
}

int rot_tables(vh_model *m, const vx_ragged &b, const MixActs &a) {
    const MixModel &x = *m->mix;
    for (size_t i = 0; i < x.rotations.size(); i++)
        VXC(vx_rotary_table(m->be, b.token_pos, b.rows, (int)x.rotations[i].freqs.size(), x.rotations[i].d_freqs, x.rotations[i].factor,
                            (float *)rot_table(x, a, b.rows, (int)i)));
    return VH_OK;
}

int embed(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, float *out) {
    const MixModel &x = *m->mix;
    if (!x.pairs) {
        VXC(vx_embedding(m->be, d_tokens, b.rows, m->embedding, out, m->cfg.vocab, m->cfg.hidden));
        return VH_OK;
    }
    vx_pair_embedding_args e;
    memset(&e, 0, sizeof e);
    e.cols = m->cfg.hidden, e.vocab = m->cfg.vocab, e.buckets = x.buckets, e.mul_prev = x.mul_prev, e.mul_cur = x.mul_cur;
    e.tokens = d_tokens, e.embed = m->embedding, e.pairs = x.pairs, e.token_pool = x.token_pool, e.out = out;
    VXC(vx_pair_embedding(m->be, &b, &e));
    return VH_OK;
}

// the experts of every row, from the router's logits z (float32, in slices)
int run_router(vh_model *m, const MixLayer &l, int rows, const MixActs &a, const float *z, int slices, int ldz) {
    const ExpertMlp &e = l.moe;
    vx_route_args r;
    memset(&r, 0, sizeof r);
    r.rows = rows, r.experts = e.experts, r.top = e.top, r.groups = e.groups, r.keep = e.keep, r.shared = e.shared;
    r.tile_rows = vx_route_tile_rows(m->mix->act, rows, e.experts, e.top);
    r.z = z + e.router_col, r.z_slices = slices, r.ldz = ldz, r.z_stride = (int64_t)rows * ldz;
    r.bias = e.router_bias, r.softmax = e.softmax;
    r.correction = e.correction, r.weights = a.e_weights, r.places = a.e_places, r.order = a.e_order, r.tiles = a.e_tiles;
    VXC(vx_route(m->be, &r));
    return VH_OK;
}

// a.h -> the chosen experts' results in a.e_out, by place
int run_experts(vh_model *m, const MixLayer &l, int rows, const MixActs &a) {
    const MixModel &x = *m->mix;
    const ExpertMlp &e = l.moe;
    vx_experts_args g;
    memset(&g, 0, sizeof g);
    g.rows = rows, g.experts = e.experts, g.shared = e.shared;
    g.tile_rows = vx_route_tile_rows(m->mix->act, rows, e.experts, e.top);
    g.max_tiles = vx_route_max_tiles(rows, e.experts, e.top, e.shared, g.tile_rows);
    g.tiles = a.e_tiles;
    g.kind = e.relu2 ? VX_LIN_RELU2 : VX_LIN_SWIGLU, g.a = a.h, g.lda = pad_to(m->cfg.hidden, 64), g.a_rows = a.e_order;
    g.w = e.gate_up.w, g.n = e.gate_up.n, g.k = e.gate_up.k, g.w_shared = e.shared_gate_up.w, g.n_shared = e.shared_gate_up.n, g.k_shared = e.shared_gate_up.k;
    g.glu_limit = e.limit, g.shared_limit = e.shared_limit, g.glu_alpha = e.alpha, g.glu_add = e.add;
    g.out = a.e_act, g.ldo = std::max(e.ff_pad, e.shared_pad), g.cols = e.ff_pad, g.cols_shared = e.shared_pad;
    VXC(vx_linear_experts(m->be, x.act, &g));
    g.kind = VX_LIN_PLAIN, g.a = a.e_act, g.lda = g.ldo, g.a_rows = nullptr;
    g.w = e.down.w, g.n = e.down.n, g.k = e.down.k, g.w_shared = e.shared_down.w, g.n_shared = e.shared_down.n, g.k_shared = e.shared_down.k;
    g.out = a.e_out, g.ldo = g.cols = g.cols_shared = e.down.n;
    VXC(vx_linear_experts(m->be, x.act, &g));
    return VH_OK;
}

int run_out(vh_model *m, const MixLayer &l, int rows, const MixActs &a, int *slices) {
    *slices = vx_linear_slices(m->be, l.out.n, l.out.k, rows);
    vx_linear_out o = plain(a.y, 1, l.out.n, l.out.n, *slices);
    VXC(vx_linear(m->be, m->mix->act, a.cat, l.out.k, l.out.w, l.out.n, l.out.k, rows, &o));
    return VH_OK;
}

// A layer's one mixer: a.h -> its output as `slices` partial sums in a.y; where experts stand beside it, their choice as well.
int run_mixer(vh_model *m, const LayerRun &r, const vx_ragged &b, const MixActs &a, int *slices) {
    const MixModel &x = *m->mix;
    const MixLayer &l = x.layers[r.layer];
    const size_t es = esize(x);
    const int rows = b.rows, width_pad = pad_to(m->cfg.hidden, 64), ldc = l.out.k;
    const bool beside = l.has_experts && !l.moe.router.w;
    if (l.has_forget) {
        const ForgetMixer &t = l.forget;
        const int qs = t.heads * t.dim_pad, vs = t.heads * t.v_pad;
        vx_linear_out o = plain(a.proj, 0, qs + vs, qs + vs, 1);
        o.kind = VX_LIN_FORGET;
        o.split = qs + vs, o.silu_cols = qs, o.out2 = a.y, o.ldo2 = qs, o.bias = t.bias, o.keep = t.keep;
        VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
        vx_forget_args d;
        memset(&d, 0, sizeof d);
        d.heads = t.heads, d.dim = t.dim_pad, d.vdim = t.v_pad;
        d.q = a.proj, d.v = at(a.proj, qs, es), d.g = a.y, d.ldq = d.ldv = qs + vs, d.ldg = qs;
        d.state = r.state, d.out = a.o, d.ldo = vs;
        VXC(vx_forget_attn(m->be, x.act, &b, &d));
        VXC(vx_head_norm(m->be, x.act, a.o, vs, t.norm, x.eps, rows, t.heads, t.v_pad, t.vdim, a.cat, ldc));
        return run_out(m, l, rows, a, slices);
    }
    if (l.has_decay) {
        const DecayMixer &t = l.decay;
        const int side = l.in.n - t.split, vs = t.heads * t.v_pad;
        vx_linear_out o = plain(a.proj, 0, t.split, t.split, 1);
        o.kind = VX_LIN_SILU;
        o.split = t.split, o.out2 = a.y, o.ldo2 = side;
        VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
        if (beside) VHC(run_router(m, l, rows, a, a.y, 1, side));
        vx_decay_args d;
        memset(&d, 0, sizeof d);
        d.heads = t.heads, d.dim = t.dim_pad, d.vdim = t.v_pad, d.decay = t.decay;
        d.q = a.proj, d.k = at(a.proj, (size_t)t.heads * t.dim_pad, es), d.v = at(a.proj, (size_t)2 * t.heads * t.dim_pad, es);
        d.ldq = d.ldk = d.ldv = t.split;
        d.state = r.state, d.out = a.o, d.ldo = vs;
        VXC(vx_decay_attn(m->be, x.act, &b, &d));
        VXC(vx_gated_norm(m->be, x.act, a.o, vs, a.y + t.g_col, side, t.norm, x.eps, rows, vs, t.heads * t.vdim, a.cat, ldc));
        return run_out(m, l, rows, a, slices);
    }
    const AttnMixer &t = l.attn;
    *slices = vx_linear_slices(m->be, l.in.n, l.in.k, rows);
    vx_linear_out o = plain(a.y, 1, l.in.n, l.in.n, *slices);
    VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
    if (beside) VHC(run_router(m, l, rows, a, a.y, *slices, l.in.n));
    vx_heads_args h;
    memset(&h, 0, sizeof h);
    h.q_heads = t.heads * t.maps, h.dim = t.k_dim, h.v_dim = t.v_dim;
    h.y = a.y, h.y_slices = *slices, h.ldy = l.in.n, h.y_stride = (int64_t)rows * l.in.n, h.bias = t.in_bias;
    h.q_col = t.q_col, h.k_col = t.k_col, h.v_col = t.v_col;
    if (t.rotation >= 0) h.rot_pairs = (int)x.rotations[t.rotation].freqs.size(), h.rot_tab = rot_table(x, a, rows, t.rotation);
    if (t.kv_from < 0) h.k_heads = t.kv_heads * t.maps, h.v_heads = t.kv_heads;
    h.norm = t.row_norm ? 2 : t.norm, h.eps = x.eps, h.w_q = t.norm_q, h.w_k = t.norm_k;
    h.q = a.proj, h.ldq = by_heads_ldq(t), h.pool = r.kv;
    VXC(vx_heads_store(m->be, x.act, &b, &h));
    if (t.heads * t.v_dim < ldc) VXC(vx_fill_zero(m->be, a.cat, (size_t)rows * ldc * es));
    vx_attn_args at_;
    memset(&at_, 0, sizeof at_);
    at_.heads = t.heads, at_.kv_heads = t.kv_heads, at_.k_dim = t.k_dim, at_.v_dim = t.v_dim, at_.scale = t.scale, at_.sink = t.sink;
    at_.window = t.window, at_.chunk = t.chunk, at_.softcap = t.softcap;
    at_.slopes = t.slopes, at_.talk = t.talk;
    at_.maps = t.maps, at_.diff_lambda = t.diff_lambda, at_.diff_scale = t.diff_scale, at_.diff_eps = x.eps;
    at_.q = a.proj, at_.ldq = h.ldq, at_.pool = r.kv, at_.out_scale = 1.f, at_.out = a.cat, at_.ldo = ldc;
    VXC(vx_attn_ragged(m->be, x.act, &b, &at_));
    return run_out(m, l, rows, a, slices);
}

// mixers of one layer run: a.h -> the sublayer's output as `slices` partial sums in a.y
int run_mixers(vh_model *m, const LayerRun &r, const vx_ragged &b, const MixActs &a, int *slices) {
    const MixModel &x = *m->mix;
    const MixLayer &l = x.layers[r.layer];
    const size_t es = esize(x);
    const int rows = b.rows, width_pad = pad_to(m->cfg.hidden, 64), ldp = l.in.n, ldc = l.out.k;
    vx_linear_out o = plain(a.proj, 0, ldp, ldp, 1);
    if (l.has_attn) {
        o.kind = VX_LIN_KV;
        o.k_col = l.attn.k_col, o.v_col = l.attn.v_col, o.kv_heads = l.attn.kv_heads, o.k_dim = l.attn.k_dim, o.v_dim = l.attn.v_dim;
        o.block_size = b.block_size, o.pool = r.kv, o.slot_mapping = b.slot_mapping;
    }
    VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
    const int attn_cols = l.has_attn ? l.attn.heads * l.attn.v_dim : 0;
    if (!l.has_scan && attn_cols < ldc) VXC(vx_fill_zero(m->be, a.cat, (size_t)rows * ldc * es));
    if (l.has_scan) {
        const ScanMixer &s = l.scan;
        vx_conv_args cv;
        memset(&cv, 0, sizeof cv);
        cv.channels = s.channels, cv.taps = s.taps;
        cv.x = at(a.proj, s.x_col, es), cv.ldx = ldp;
        cv.w = s.conv_w, cv.b = s.conv_b, cv.state = r.conv;
        cv.out = a.xc, cv.ldo = s.x.k;
        VXC(vx_conv_silu(m->be, x.act, &b, &cv));
        o = plain(a.dtr, 0, s.dt_pad, s.dt_pad, 1);
        o.kind = VX_LIN_SPLIT;
        o.split = s.dt_pad, o.out2 = a.bc, o.ldo2 = 2 * s.pad;
        VXC(vx_linear(m->be, x.act, a.xc, s.x.k, s.x.w, s.x.n, s.x.k, rows, &o));
        o = plain(a.dt, 1, s.dt.n, s.channels, 1);
        o.kind = VX_LIN_SOFTPLUS;
        o.bias = s.dt_bias;
        VXC(vx_linear(m->be, x.act, a.dtr, s.dt_pad, s.dt.w, s.dt.n, s.dt.k, rows, &o));
        vx_scan_args sc;
        memset(&sc, 0, sizeof sc);
        sc.channels = s.channels, sc.states = s.states;
        sc.a2 = s.a2, sc.d = s.d;
        sc.x = a.xc, sc.ldx = s.x.k;
        sc.z = at(a.proj, s.z_col, es), sc.ldz = ldp;
        sc.dt = a.dt, sc.lddt = s.dt.n, sc.bc = a.bc;
        sc.state = r.state, sc.out_scale = s.out_scale;
        sc.out = at(a.cat, attn_cols, es), sc.ldo = ldc, sc.out_cols = ldc - attn_cols;
        VXC(vx_selective_scan(m->be, x.act, &b, &sc));
    }
    if (l.has_attn) {
        const AttnMixer &t = l.attn;
        vx_attn_args at_;
        memset(&at_, 0, sizeof at_);
        at_.heads = t.heads, at_.kv_heads = t.kv_heads, at_.k_dim = t.k_dim, at_.v_dim = t.v_dim;
        at_.scale = t.scale, at_.temp_coef = t.temp_coef, at_.temp_every = t.temp_every;
        at_.bias = t.bias, at_.bias_len = t.bias_len;
        at_.q = at(a.proj, t.q_col, es), at_.ldq = ldp;
        at_.gate = t.gate ? at(a.proj, t.g_col, es) : nullptr, at_.ldg = ldp;
        at_.pool = r.kv, at_.out_scale = t.out_scale, at_.out = a.cat, at_.ldo = ldc;
        VXC(vx_attn_ragged(m->be, x.act, &b, &at_));
    }
    return run_out(m, l, rows, a, slices);
}

// latent attention of one layer run: a.h -> the sublayer's output as `slices` partial sums in a.y
int run_latent(vh_model *m, const LayerRun &r, const vx_ragged &b, const MixActs &a, const MixExpand *ex, int *slices) {
    const MixModel &x = *m->mix;
    const MixLayer &l = x.layers[r.layer];
    const LatentMixer &t = l.latent;
    const size_t es = esize(x);
    const int rows = b.rows, width_pad = pad_to(m->cfg.hidden, 64), q_cols = t.heads * t.head_cols, ldc = l.out.k;
    const float *tab = rot_table(x, a, rows, t.rotation);
    const auto heads_out = [&]() {  // the queries' projection: heads, their last part turned
        vx_linear_out o = plain(a.proj, 0, q_cols, q_cols, 1);
        if (tab) {
            o.kind = VX_LIN_ROTARY;
            o.split = q_cols, o.rot_stride = t.head_cols, o.rot_first = t.dim_pad, o.rot_pairs = t.rot_dim / 2, o.rot_tab = tab;
        }
        return o;
    };
    vx_latent_store_args st;
    memset(&st, 0, sizeof st);
    st.y = a.y, st.y_slices = 1, st.eps = x.eps, st.rot_tab = tab;
    if (t.kv_from < 0) st.rank = t.rank, st.rot_dim = t.rot_dim, st.w_c = t.norm_c, st.pool = r.kv;
    if (t.q_rank > 0) {  // query latent and key latent in one float32 projection
        *slices = vx_linear_slices(m->be, l.in.n, l.in.k, rows);
        vx_linear_out o = plain(a.y, 1, l.in.n, l.in.n, *slices);
        VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
        st.y_slices = *slices, st.ldy = l.in.n, st.y_stride = (int64_t)rows * l.in.n;
        st.c_col = t.c_col, st.kr_col = t.kr_col, st.q_rank = t.q_rank, st.w_q = t.norm_q, st.q_out = a.qc, st.ldq = t.q_up.k;
        VXC(vx_latent_store(m->be, x.act, &b, &st));
        o = heads_out();
        VXC(vx_linear(m->be, x.act, a.qc, t.q_up.k, t.q_up.w, t.q_up.n, t.q_up.k, rows, &o));
    } else {
        vx_linear_out o = heads_out();
        if (t.kv_cols > 0) {
            if (!tab) o.kind = VX_LIN_SPLIT, o.split = q_cols;
            o.out2 = a.y, o.ldo2 = t.kv_cols;
        }
        VXC(vx_linear(m->be, x.act, a.h, width_pad, l.in.w, l.in.n, l.in.k, rows, &o));
        st.ldy = t.kv_cols, st.c_col = t.c_col, st.kr_col = t.kr_col;
        if (st.rank > 0) VXC(vx_latent_store(m->be, x.act, &b, &st));
    }
    if (t.heads * t.v_pad < ldc) VXC(vx_fill_zero(m->be, a.cat, (size_t)rows * ldc * es));
    // sequences with many rows: keys and values of all their tokens spelled out, once for all rows and heads
    const int k_cols = t.heads * t.dim_pad;
    const void *values = at(t.expand.w, (size_t)k_cols * t.rank_pad, 2);
    const int many = ex && ex->rows > 0 ? t.expand_rows : 0;
    bool few = many == 0;
    if (many > 0)
        for (int s = 0; s < b.n_seqs; s++) few = few || b.q_lens[s] < many;
    if (few) {
        vx_linear_out o = plain(a.qa, 0, t.heads * t.rank_pad, t.rank_pad, 1);
        o.groups = t.heads, o.a_group = t.head_cols, o.out_group = t.rank_pad;
        VXC(vx_linear(m->be, x.act, a.proj, q_cols, t.absorb.w, t.rank_pad, t.dim_pad, rows, &o));
        vx_latent_attn_args at_;
        memset(&at_, 0, sizeof at_);
        at_.heads = t.heads, at_.rank = t.rank, at_.rot_dim = t.rot_dim, at_.scale = t.scale, at_.sink = t.sink;
        at_.q = a.qa, at_.ldq = t.heads * t.rank_pad;
        at_.qr = at(a.proj, t.dim_pad, es), at_.ldqr = q_cols, at_.qr_stride = t.head_cols;
        at_.pool = r.kv, at_.out = a.lo, at_.ldo = t.heads * t.rank_pad, at_.max_rows = many > 0 ? many - 1 : 0;
        VXC(vx_attn_latent(m->be, x.act, &b, &at_));
        o = plain(a.cat, 0, ldc, t.v_pad, 1);
        o.groups = t.heads, o.a_group = t.rank_pad, o.out_group = t.v_pad;
        VXC(vx_linear(m->be, x.act, a.lo, t.heads * t.rank_pad, values, t.v_pad, t.rank_pad, rows, &o));
    }
    if (many > 0) {
        vx_linear_out o = plain(a.proj, 0, k_cols, k_cols, 1);  // (every column leaves for the pool)
        o.kind = VX_LIN_KV;
        o.kv_heads = t.heads, o.k_dim = t.head_cols, o.k_used = t.dim_pad, o.v_dim = t.v_pad, o.v_col = k_cols;
        o.block_size = b.block_size, o.pool = ex->kv, o.a_rows = ex->slots;
        VXC(vx_linear(m->be, x.act, r.kv, t.row, t.expand.w, k_cols, t.rank_pad, ex->rows, &o));
        o.kind = VX_LIN_V, o.v_col = 0, o.cols = o.ldo = t.heads * t.v_pad;
        VXC(vx_linear(m->be, x.act, r.kv, t.row, values, t.heads * t.v_pad, t.rank_pad, ex->rows, &o));
        VXC(vx_latent_spread(m->be, x.act, r.kv, t.rank, t.head_cols - t.dim_pad, ex->slots, ex->rows, ex->kv, t.heads, t.head_cols, t.v_pad, b.block_size,
                             t.dim_pad));
        vx_ragged eb = b;
        eb.table_rows = ex->table_rows, eb.block_tables = ex->tables, eb.max_blocks = ex->max_blocks;
        eb.max_kv_len = std::min(b.max_kv_len, ex->max_blocks * b.block_size);
        vx_attn_args at_;
        memset(&at_, 0, sizeof at_);
        at_.heads = at_.kv_heads = t.heads, at_.k_dim = t.head_cols, at_.v_dim = t.v_pad, at_.scale = t.scale, at_.sink = t.sink;
        at_.q = a.proj, at_.ldq = q_cols, at_.pool = ex->kv, at_.out_scale = 1.f, at_.out = a.cat, at_.ldo = ldc, at_.min_rows = many;
        VXC(vx_attn_ragged(m->be, x.act, &eb, &at_));
    }
    return run_out(m, l, rows, a, slices);
}

int run_mlp(vh_model *m, const MixLayer &l, int rows, const MixActs &a, int *slices) {
    const MixModel &x = *m->mix;
    const int width_pad = pad_to(m->cfg.hidden, 64);
    const int cut = l.poly ? vx_linear_slices(m->be, l.gate_up.n, l.gate_up.k, rows) : 1;
    vx_linear_out o = plain(l.poly ? a.z : a.act, cut > 1, l.ff_pad, l.ff_pad, cut);
    if (!l.poly) o.kind = l.relu2 ? VX_LIN_RELU2 : VX_LIN_SWIGLU;
    o.bias = l.up_bias;
    VXC(vx_linear(m->be, x.act, a.h, width_pad, l.gate_up.w, l.gate_up.n, l.gate_up.k, rows, &o));
    if (l.poly)
        VXC(vx_poly_norm(m->be, x.act, a.z, l.ff_pad, cut > 1 ? cut : 0, (int64_t)rows * l.ff_pad, rows, l.ff, l.poly, x.eps, a.act, l.ff_pad));
    *slices = vx_linear_slices(m->be, l.down.n, l.down.k, rows);
    o = plain(a.y, 1, l.down.n, l.down.n, *slices);
    VXC(vx_linear(m->be, x.act, a.act, l.ff_pad, l.down.w, l.down.n, l.down.k, rows, &o));
    return VH_OK;
}

}  // namespace

namespace {

int head_logits(vh_model *m, const MixActs &a, int n, float *logits) {
    const MixModel &x = *m->mix;
    vx_linear_out o = plain(logits, 1, m->cfg.vocab, m->cfg.vocab, 1);
    o.softcap = x.softcap, o.mult = x.logit_mult;
    VXC(vx_linear(m->be, x.act, a.h, pad_to(m->cfg.hidden, 64), x.head.w, x.head.n, x.head.k, n, &o));
    return VH_OK;
}

// Layers whose norms precede the sublayers: the seams add what the last one left, normed, and norm what the next one reads.
int forward_pre_norm(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const int32_t *want, int n_want) {
    const MixModel &x = *m->mix;
    const vh_config &c = m->cfg;
    const int rows = b.rows, width_pad = pad_to(c.hidden, 64);
    float *emb = a.emb ? a.emb : a.x;
    VHC(embed(m, b, d_tokens, emb));
    VHC(rot_tables(m, b, a));
    vx_residual_norm_args s;
    memset(&s, 0, sizeof s);
    s.rows = rows, s.cols = c.hidden, s.x_in = emb, s.x_out = a.x, s.mult = x.mult, s.eps = x.eps, s.out = a.h, s.ldo = width_pad;
    bool pending = false;         // a sublayer's output waits in a.y, for the norm `post` (or none)
    const float *post = nullptr;
    const MixLayer *beside = nullptr;  // whose experts' results wait in a.e_out
    int slices = 1;
    auto take = [&]() {
        s.y = pending ? a.y : nullptr;
        s.w_post = post, s.y_slices = slices, s.ldy = pad_to(c.hidden, 16), s.y_stride = (int64_t)rows * s.ldy;
        s.e_rows = nullptr, s.y_bias = nullptr;
        if (!beside) return;
        s.y_bias = beside->out_bias;
        if (!beside->has_experts) return;
        const ExpertMlp &e = beside->moe;
        s.e_rows = a.e_out, s.lde = e.down.n, s.e_top = e.top, s.e_shared = e.shared ? rows * e.top : -1;
        s.e_places = a.e_places, s.e_weights = a.e_weights;
    };
    auto seam = [&](const float *next, const float *add) {
        take();
        s.add = add, s.w_pre = next;
        const int rc = vx_residual_norm(m->be, x.act, &s);
        s.x_in = a.x;
        return rc;
    };
    for (const LayerRun &r : x.runs) {
        const MixLayer &l = x.layers[r.layer];
        VXC(seam(l.norm1, r.add_embedding ? emb : nullptr));
        pending = true;
        if (!l.norm1b) {
            VHC(run_mixer(m, r, b, a, &slices));
            if (l.has_experts) VHC(run_experts(m, l, rows, a));
            post = nullptr, beside = &l;
            continue;
        }
        beside = nullptr;
        VHC(run_mixers(m, r, b, a, &slices));
        post = l.norm1b;
        if (l.has_mlp) {
            VXC(seam(l.norm2, nullptr));
            VHC(run_mlp(m, l, rows, a, &slices));
            post = l.norm2b;
        }
    }
    if (n_want == 0) return VH_OK;
    take();
    s.rows = n_want, s.row_idx = want, s.x_out = nullptr;
    s.add = nullptr, s.w_pre = m->final_norm;
    VXC(vx_residual_norm(m->be, x.act, &s));
    return VH_OK;
}

// Layers whose norms follow the residual sums; the sublayers read the stream itself, and every layer's result is kept for the
// averages of those behind it.
int forward_post_norm(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const MixExpand *ex, const int32_t *want,
                      int n_want) {
    const MixModel &x = *m->mix;
    const vh_config &c = m->cfg;
    const int rows = b.rows, n_runs = (int)x.runs.size();
    VHC(embed(m, b, d_tokens, a.hist));
    VHC(rot_tables(m, b, a));
    vx_post_norm_args s;
    memset(&s, 0, sizeof s);
    s.rows = rows, s.cols = c.hidden, s.x_in = a.hist, s.eps = x.eps, s.alpha = x.alpha, s.out = a.h, s.ldo = pad_to(c.hidden, 64);
    s.hist = a.hist, s.hist_stride = (int64_t)rows * c.hidden, s.keep = 1;
    VXC(vx_post_norm(m->be, x.act, &s));
    s.x_out = a.x, s.y = a.y, s.ldy = pad_to(c.hidden, 16), s.y_stride = (int64_t)rows * s.ldy;
    for (int i = 0; i < n_runs; i++) {
        const MixLayer &l = x.layers[x.runs[i].layer];
        VHC(run_latent(m, x.runs[i], b, a, ex, &s.y_slices));
        s.w = l.norm1;
        if (l.has_mlp) {
            VXC(vx_post_norm(m->be, x.act, &s));
            s.x_in = a.x;
            VHC(run_mlp(m, l, rows, a, &s.y_slices));
            s.w = l.norm2;
        }
        s.avg = l.depth_avg, s.n_avg = l.depth_avg ? i + 2 : 0;
        if (i + 1 == n_runs) {  // the rows whose logits are asked for alone, with the final norm
            if (n_want == 0) return VH_OK;
            s.rows = n_want, s.row_idx = want, s.keep = 0, s.x_out = nullptr, s.w_pre = m->final_norm;
        }
        VXC(vx_post_norm(m->be, x.act, &s));
        s.x_in = a.x, s.n_avg = 0;
    }
    return VH_OK;
}

// Layers whose sublayers read the stream itself and are layer-normed before they join it.
int forward_branch_norm(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const int32_t *want, int n_want) {
    const MixModel &x = *m->mix;
    const vh_config &c = m->cfg;
    const int rows = b.rows, n_runs = (int)x.runs.size();
    VHC(rot_tables(m, b, a));
    vx_branch_norm_args s;
    memset(&s, 0, sizeof s);
    s.rows = rows, s.cols = c.hidden, s.eps = x.eps, s.x_out = a.x, s.out = a.h, s.ldo = pad_to(c.hidden, 64);
    s.x_in = m->embedding, s.tokens = d_tokens, s.token_pos = b.token_pos, s.positions = x.positions, s.w_pre = x.emb_norm, s.b_pre = x.emb_norm_b;
    VXC(vx_branch_norm(m->be, x.act, &s));
    s.x_in = a.x, s.tokens = nullptr, s.w_pre = s.b_pre = nullptr;
    s.ldy = pad_to(c.hidden, 16), s.y_stride = (int64_t)rows * s.ldy;
    const auto join = [&](const float *w, const float *bias, bool last) {
        s.w = w, s.b = bias;
        if (last) s.rows = n_want, s.row_idx = want, s.x_out = nullptr, s.w_pre = m->final_norm, s.b_pre = x.final_norm_b;
        return vx_branch_norm(m->be, x.act, &s);
    };
    for (int i = 0; i < n_runs; i++) {
        const MixLayer &l = x.layers[x.runs[i].layer];
        const bool last = i + 1 == n_runs, ff = l.has_mlp || l.has_experts;
        VHC(run_mixer(m, x.runs[i], b, a, &s.y_slices));
        s.y = a.y, s.y_bias = l.out_bias, s.e_rows = nullptr;
        if (last && n_want == 0 && !ff) return VH_OK;
        VXC(join(l.norm1, l.norm1b, last && !ff));
        if (!ff) continue;
        if (last && n_want == 0) return VH_OK;  // (nothing behind the last layer's mixer is kept)
        if (l.has_mlp) {
            VHC(run_mlp(m, l, rows, a, &s.y_slices));
            s.y_bias = l.down_bias;
        } else {
            const ExpertMlp &e = l.moe;
            const int cut = vx_linear_slices(m->be, e.router.n, e.router.k, rows);
            vx_linear_out o = plain(a.y, 1, e.router.n, e.router.n, cut);
            VXC(vx_linear(m->be, x.act, a.h, pad_to(c.hidden, 64), e.router.w, e.router.n, e.router.k, rows, &o));
            VHC(run_router(m, l, rows, a, a.y, cut, e.router.n));
            VHC(run_experts(m, l, rows, a));
            s.y = s.y_bias = nullptr;
            s.e_rows = a.e_out, s.lde = e.down.n, s.e_top = e.top, s.e_places = a.e_places, s.e_weights = a.e_weights;
        }
        VXC(join(l.norm2, l.norm2b, last));
    }
    return VH_OK;
}

}  // namespace

int mix_forward(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const MixExpand *ex, const int32_t *want,
                int n_want, float *logits) {
    if (b.rows > a.rows) return fail("internal: %d rows, activations for %d", b.rows, a.rows);
    VHC(m->mix->branch_norm ? forward_branch_norm(m, b, d_tokens, a, want, n_want)
        : m->mix->post_norm ? forward_post_norm(m, b, d_tokens, a, ex, want, n_want) : forward_pre_norm(m, b, d_tokens, a, want, n_want));
    return n_want > 0 ? head_logits(m, a, n_want, logits) : (int)VH_OK;
}

namespace {

// The part of a step that spells keys and values out: lens / tables of the sequences after it. Nothing when no sequence brings
// enough rows, or when the spelled-out keys would take too much memory.
int plan_expand(vh_model *m, int n_seqs, const int32_t *q_lens, const std::vector<int> &lens, const std::vector<std::vector<int32_t>> &tables,
                MixExpand *ex) {
    const MixModel &x = *m->mix;
    const int bs = m->cfg.block_size;
    if (x.expand_rows <= 0) return VH_OK;
    int64_t blocks = 0, most = 0;
    for (int i = 0; i < n_seqs; i++)
        if (q_lens[i] >= x.expand_rows) {
            const int64_t n = (lens[i] + bs - 1) / bs;
            blocks += n, most = std::max(most, n);
        }
    size_t per_block = 0;
    for (const MixLayer &l : x.layers)
        if (l.has_latent && l.latent.expand_rows > 0)
            per_block = std::max(per_block, vx_kv_block_elems(bs, l.latent.heads, l.latent.head_cols, l.latent.v_pad) * esize(x));
    if (blocks == 0 || blocks * bs > (1 << 22) || blocks * per_block > ((size_t)8 << 30)) return VH_OK;
    ex->rows = (int)blocks * bs, ex->max_blocks = (int)most;
    std::vector<int32_t> up((size_t)ex->rows + (size_t)n_seqs * most + n_seqs);
    int32_t *slots = up.data(), *tab = slots + ex->rows, *ids = tab + (size_t)n_seqs * most;
    int64_t at = 0;
    for (int i = 0; i < n_seqs; i++) {
        ids[i] = i;
        for (int64_t k = 0; k < most; k++) tab[i * most + k] = 0;
        if (q_lens[i] < x.expand_rows) continue;
        const int n = (lens[i] + bs - 1) / bs;
        for (int k = 0; k < n; k++, at++) {
            tab[i * most + k] = (int32_t)at;
            for (int t = 0; t < bs; t++) slots[at * bs + t] = tables[i][k] * bs + t;  // (behind the last token: finite, not seen)
        }
    }
    ex->kv = vx_alloc(m->be, blocks * per_block);
    int32_t *d = (int32_t *)vx_alloc(m->be, up.size() * 4);
    if (!ex->kv || !d) return fail("spelled-out keys: %s", vx_last_error());
    VXC(vx_to_device(m->be, d, up.data(), up.size() * 4));
    ex->slots = d, ex->tables = d + ex->rows, ex->table_rows = ex->tables + (size_t)n_seqs * most;
    return VH_OK;
}

}  // namespace

int mix_step(vh_model *m, int n_seqs, const int64_t *seq_ids, const int32_t *q_lens, const int32_t *tokens, int n_want,
             const int32_t *want_rows, float *logits_out, int32_t *argmax_out) {
    const vh_config &c = m->cfg;
    vx_backend *be = m->be;
    if (n_seqs > c.max_seqs) return fail("%d sequences in one step, the model holds %d", n_seqs, c.max_seqs);
    if (n_seqs > 1024) return fail("%d sequences in one step (at most 1024)", n_seqs);
    std::set<int64_t> seen;
    int64_t total = 0;
    bool one_each = true;
    for (int i = 0; i < n_seqs; i++) {
        if (q_lens[i] < 1) return fail("sequence %lld brings no tokens", (long long)seq_ids[i]);
        if (!seen.insert(seq_ids[i]).second) return fail("sequence %lld appears twice", (long long)seq_ids[i]);
        total += q_lens[i];
        one_each = one_each && q_lens[i] == 1;
    }
    if (total > (1 << 20)) return fail("%lld tokens in one step", (long long)total);
    const int T = (int)total;
    for (int t = 0; t < T; t++)
        if (tokens[t] < 0 || tokens[t] >= c.vocab) return fail("token %d out of range", tokens[t]);
    if (n_want > T) return fail("%d rows wanted of %d", n_want, T);
    for (int w = 0; w < n_want; w++)
        if (want_rows[w] < 0 || want_rows[w] >= T) return fail("wanted row %d of %d", want_rows[w], T);
    std::vector<int32_t> slots(n_seqs), pos(n_seqs);
    std::vector<int> lens(n_seqs);
    std::vector<std::vector<int32_t>> seq_tables(n_seqs);  // of the sequences that may be spelled out
    int max_kv = 1;
    {
        std::lock_guard<std::mutex> g(m->pool.mu);
        int64_t need = 0;
        size_t fresh = 0;
        for (int i = 0; i < n_seqs; i++) {  // nothing changes unless the whole step has room
            const SeqState *s = find_seq(m, seq_ids[i]);
            fresh += s == nullptr;
            const int have = s ? (int)s->table.size() : 0, len = (s ? s->seq_len : 0) + q_lens[i];
            const int blocks = (len - 1) / c.block_size + 1;
            if (blocks > c.max_blocks_per_seq)
                return fail("sequence %lld: %d tokens need %d blocks, max_blocks_per_seq is %d", (long long)seq_ids[i], len, blocks,
                            c.max_blocks_per_seq);
            if (m->mix->max_positions > 0 && len > m->mix->max_positions)
                return fail("sequence %lld: %d tokens, the model has %d positions", (long long)seq_ids[i], len, m->mix->max_positions);
            need += std::max(0, blocks - have);
        }
        if (fresh > m->pool.free_slots.size()) return fail("more than %d live sequences", c.max_seqs);
        if (need > (int64_t)m->pool.free_list.size())
            return fail("no free blocks: the step needs %lld, the pool has %zu", (long long)need, m->pool.free_list.size());
        for (int i = 0; i < n_seqs; i++) {
            if (!find_seq(m, seq_ids[i])) VHC(create_seq_locked(m, seq_ids[i]));
            SeqState *s = find_seq(m, seq_ids[i]);
            slots[i] = s->slot, pos[i] = s->seq_len;
            VHC(m->pool.ensure_blocks(*s, s->seq_len + q_lens[i]));
            lens[i] = s->seq_len + q_lens[i];
            max_kv = std::max(max_kv, lens[i]);
            if (m->mix->expand_rows > 0 && q_lens[i] >= m->mix->expand_rows) seq_tables[i] = s->table;
        }
        VHC(sync_pool_to_device(m));
    }
    vx_reset_pool(be);
    // one upload: tokens | slots | positions | token counts | wanted rows; behind them what vx_pack_batch derives
    const size_t up = (size_t)T + 3 * n_seqs + n_want, meta = up + (n_seqs + 1) + 2 * (size_t)T + n_seqs;
    int32_t *d = (int32_t *)vx_alloc(be, meta * 4);
    if (!d) return fail("step arrays: %s", vx_last_error());
    std::vector<int32_t> host(up);
    int32_t *h = host.data();
    memcpy(h, tokens, (size_t)T * 4), h += T;
    memcpy(h, slots.data(), (size_t)n_seqs * 4), h += n_seqs;
    memcpy(h, pos.data(), (size_t)n_seqs * 4), h += n_seqs;
    memcpy(h, q_lens, (size_t)n_seqs * 4), h += n_seqs;
    if (n_want) memcpy(h, want_rows, (size_t)n_want * 4);
    VXC(vx_to_device(be, d, host.data(), up * 4));
    int32_t *d_tok = d, *d_slots = d + T, *d_pos = d_slots + n_seqs, *d_q = d_pos + n_seqs, *d_want = d_q + n_seqs;
    int32_t *d_cu = d + up, *d_tp = d_cu + n_seqs + 1, *d_sm = d_tp + T, *d_kvl = d_sm + T;
    MixActs acts = m->mix->perm;
    if (T > acts.rows) VHC(alloc_acts(m, T, false, [&](size_t n) { return vx_alloc(be, n); }, &acts));
    float *logits = m->logits;
    if (n_want > c.max_batch) {
        logits = (float *)vx_alloc(be, (size_t)n_want * c.vocab * 4);
        if (!logits) return fail("logits of %d rows: %s", n_want, vx_last_error());
    }
    MixExpand ex;
    if (!one_each) VHC(plan_expand(m, n_seqs, q_lens, lens, seq_tables, &ex));
    VXC(vx_pack_batch(be, d_slots, d_pos, one_each ? nullptr : d_q, n_seqs, T, m->d_tables, c.max_blocks_per_seq, m->d_num_blocks,
                      m->d_free, m->d_free_count, c.block_size, d_cu, d_tp, d_sm, d_kvl, m->d_status));
    const vx_ragged b{T, n_seqs, one_each ? nullptr : q_lens, max_kv, d_cu, d_tp, d_sm, d_slots, d_kvl, m->d_tables, c.max_blocks_per_seq,
                      c.block_size};
    VHC(mix_forward(m, b, d_tok, acts, ex.rows > 0 ? &ex : nullptr, n_want ? d_want : nullptr, n_want, logits));
    if (n_want > 0 && argmax_out) {
        int32_t *d_am = n_want <= c.max_batch ? m->d_next : (int32_t *)vx_alloc(be, (size_t)n_want * 4);
        if (!d_am) return fail("arg-max rows: %s", vx_last_error());
        VXC(vx_argmax_rows(be, logits, n_want, c.vocab, d_am));
        VXC(vx_to_host(be, argmax_out, d_am, (size_t)n_want * 4));
    }
    if (n_want > 0 && logits_out) VXC(vx_to_host(be, logits_out, logits, (size_t)n_want * c.vocab * 4));
    VXC(vx_sync(be));
    std::lock_guard<std::mutex> g(m->pool.mu);
    for (int i = 0; i < n_seqs; i++)
        if (SeqState *s = find_seq(m, seq_ids[i])) s->seq_len = pos[i] + q_lens[i];
    return VH_OK;
}

}  // namespace vh
