// Mixer programs: the executor of models whose layers are described one by one (model.h: MixLayer), over mixed batches.
//
// A step is a set of sequences with any number of new tokens each. Its rows run through every layer together:
//   norm | input projection (K and V leave for the paged pool on the way) | attention and / or convolution + scan | output
//   projection | norm, residual, norm | gate|up with SiLU | down | norm, residual, and the next layer's norm
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

struct Widths {
    int width_pad = 0, in = 0, out = 0, xc = 0, dtr = 0, bc = 0, dt = 0, act = 0;
};

Widths widths(const vh_model *m) {
    Widths w;
    w.width_pad = pad_to(m->cfg.hidden, 64);
    for (const MixLayer &l : m->mix->layers) {
        w.in = std::max(w.in, l.in.n);
        w.out = std::max(w.out, l.out.k);
        w.act = std::max(w.act, l.ff_pad);
        if (l.has_scan) {
            w.xc = std::max(w.xc, l.scan.x.k);
            w.dtr = std::max(w.dtr, l.scan.dt_pad);
            w.bc = std::max(w.bc, 2 * l.scan.pad);
            w.dt = std::max(w.dt, l.scan.dt.n);
        }
    }
    return w;
}

// slices x rows of float32 sublayer outputs that a step of up to `rows` rows may need
size_t slice_rows(const vh_model *m, int rows, bool up_to) {
    size_t most = 1;
    for (const MixLayer &l : m->mix->layers)
        for (const Linear *w : {&l.out, &l.down}) {
            if (!w->w) continue;
            for (int r = up_to ? 1 : rows; r <= rows; r++) most = std::max(most, (size_t)r * vx_linear_slices(m->be, w->n, w->k, r));
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
    const int cols = pad_to(m->cfg.hidden, 16);
    const bool ok = get(&a->x, R * m->cfg.hidden * 4) && get(&a->h, R * w.width_pad * es) && get(&a->proj, R * w.in * es) &&
                    get(&a->cat, R * w.out * es) && get(&a->xc, R * w.xc * es) && get(&a->dtr, R * w.dtr * es) &&
                    get(&a->bc, R * w.bc * 4) && get(&a->dt, R * w.dt * 4) && get(&a->act, R * w.act * es) &&
                    get(&a->y, slice_rows(m, rows, up_to) * cols * 4) && (!loop || get(&a->emb, R * m->cfg.hidden * 4));
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
        if (l.has_attn) {
            // (what a kernel may read beyond a sequence's tokens is a finite number from the start)
            r.kv = zeroed(vx_kv_block_elems(c.block_size, l.attn.kv_heads, l.attn.k_dim, l.attn.v_dim) * c.pool_blocks * es);
            if (!r.kv) return fail("KV pool: %s", vx_last_error());
            m->kv.back() = r.kv;
        }
        if (l.has_scan) {
            r.state = (float *)zeroed((size_t)c.max_seqs * l.scan.channels * l.scan.pad * 4);
            if (!r.state) return fail("scan state: %s", vx_last_error());
            m->adopted.push_back(r.state);
            r.conv = zeroed((size_t)c.max_seqs * (l.scan.taps - 1) * l.scan.channels * es);
            if (!r.conv) return fail("convolution state: %s", vx_last_error());
            m->adopted.push_back(r.conv);
        }
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
    *slices = vx_linear_slices(m->be, l.out.n, l.out.k, rows);
    o = plain(a.y, 1, l.out.n, l.out.n, *slices);
    VXC(vx_linear(m->be, x.act, a.cat, ldc, l.out.w, l.out.n, l.out.k, rows, &o));
    return VH_OK;
}

int run_mlp(vh_model *m, const MixLayer &l, int rows, const MixActs &a, int *slices) {
    const MixModel &x = *m->mix;
    vx_linear_out o = plain(a.act, 0, l.ff_pad, l.ff_pad, 1);
    o.kind = VX_LIN_SWIGLU;
    VXC(vx_linear(m->be, x.act, a.h, pad_to(m->cfg.hidden, 64), l.gate_up.w, l.gate_up.n, l.gate_up.k, rows, &o));
    *slices = vx_linear_slices(m->be, l.down.n, l.down.k, rows);
    o = plain(a.y, 1, l.down.n, l.down.n, *slices);
    VXC(vx_linear(m->be, x.act, a.act, l.ff_pad, l.down.w, l.down.n, l.down.k, rows, &o));
    return VH_OK;
}

}  // namespace

int mix_forward(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const int32_t *want, int n_want,
                float *logits) {
    const MixModel &x = *m->mix;
    const vh_config &c = m->cfg;
    const int rows = b.rows, width_pad = pad_to(c.hidden, 64);
    if (rows > a.rows) return fail("internal: %d rows, activations for %d", rows, a.rows);
    float *emb = a.emb ? a.emb : a.x;
    VXC(vx_embedding(m->be, d_tokens, rows, m->embedding, emb, c.vocab, c.hidden));
    // the seams between sublayers: what the last one left is normed and added, what the next one reads is normed
    vx_residual_norm_args s;
    memset(&s, 0, sizeof s);
    s.rows = rows, s.cols = c.hidden, s.x_in = emb, s.x_out = a.x, s.mult = x.mult, s.eps = x.eps, s.out = a.h, s.ldo = width_pad;
    const float *post = nullptr;  // the norm that waits for the sublayer output in a.y
    int slices = 1;
    auto seam = [&](const float *next, const float *add) {
        s.y = post ? a.y : nullptr;
        s.w_post = post, s.y_slices = slices, s.ldy = pad_to(c.hidden, 16), s.y_stride = (int64_t)rows * s.ldy;
        s.add = add, s.w_pre = next;
        const int rc = vx_residual_norm(m->be, x.act, &s);
        s.x_in = a.x;
        return rc;
    };
    for (const LayerRun &r : x.runs) {
        const MixLayer &l = x.layers[r.layer];
        VXC(seam(l.norm1, r.add_embedding ? emb : nullptr));
        VHC(run_mixers(m, r, b, a, &slices));
        post = l.norm1b;
        if (l.has_mlp) {
            VXC(seam(l.norm2, nullptr));
            VHC(run_mlp(m, l, rows, a, &slices));
            post = l.norm2b;
        }
    }
    if (n_want == 0) return VH_OK;
    s.rows = n_want, s.row_idx = want, s.x_out = nullptr;
    s.y_stride = (int64_t)rows * pad_to(c.hidden, 16);
    s.y = post ? a.y : nullptr, s.w_post = post, s.y_slices = slices, s.ldy = pad_to(c.hidden, 16);
    s.add = nullptr, s.w_pre = m->final_norm;
    VXC(vx_residual_norm(m->be, x.act, &s));
    vx_linear_out o = plain(logits, 1, c.vocab, c.vocab, 1);
    VXC(vx_linear(m->be, x.act, a.h, width_pad, x.head.w, x.head.n, x.head.k, n_want, &o));
    return VH_OK;
}

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
            max_kv = std::max(max_kv, s->seq_len + q_lens[i]);
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
    VXC(vx_pack_batch(be, d_slots, d_pos, one_each ? nullptr : d_q, n_seqs, T, m->d_tables, c.max_blocks_per_seq, m->d_num_blocks,
                      m->d_free, m->d_free_count, c.block_size, d_cu, d_tp, d_sm, d_kvl, m->d_status));
    const vx_ragged b{T, n_seqs, one_each ? nullptr : q_lens, max_kv, d_cu, d_tp, d_sm, d_slots, d_kvl, m->d_tables, c.max_blocks_per_seq,
                      c.block_size};
    VHC(mix_forward(m, b, d_tok, acts, n_want ? d_want : nullptr, n_want, logits));
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
