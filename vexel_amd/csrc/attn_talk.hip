// Paged attention whose scores are mixed across heads ahead of the softmax (vx_attn_ragged with talk), on the bfloat16 matrix cores.
//
// A workgroup takes a few rows of one sequence with all heads, and walks a piece of their keys in groups of 32. A wave owns up to four
// tiles of 16 (row, head) pairs of one K/V head each. A group takes three stages with a barrier between each:
//   scores   every wave's products Q K^T to LDS, float32 [key][row][head]
//   mix      talk * scores over 16 (key, row) pairs at a time, in place; the scores enter the product as two bfloat16 parts
//   output   every wave reads its tiles' mixed scores back, a lane eight consecutive keys of one query, for softmax and O^T = V^T P^T
// Two buffers of scores take turns, so that a group's first stage may start while other waves are still in the last one of the group
// before. Pieces of keys: partial results that a second launch merges.
#include <string.h>

#include <algorithm>

#include "attn_tiles.h"

using namespace vx;

namespace {

constexpr int MAX_WAVES = 8, MAX_TPW = 4, MAX_ROWS = 32, MAX_HEADS = 64;
constexpr int LDS_BYTES = 150 * 1024;

struct TalkArgs {
    AttnArgs a;
    int lr;               // log2 of the rows of a workgroup
    int per_kv, tiles;    // tiles of a K/V head; of all
    int hs, h8;           // floats from one row's scores to the next; heads up to a multiple of 8
    int buf;              // floats of a buffer
    int vec;              // four pairs of a lane are neighbouring heads of one row
    int many;             // sequences with several rows (else those with one)
    int items;            // (row tile, piece) pairs
};

__host__ __device__ __forceinline__ int talk_cols(int heads) { return (heads + 31) / 32 * 32 + 8; }  // LDS row of the talk matrix

// Where the score of a key (0 .. 31 of the group) lies; head and row are added.
__device__ __forceinline__ int key_at(const TalkArgs &t, int key) { return (key << t.lr) * t.hs + (key >> 3) * 16; }

template <int KD, int VD, int TPW, bool SHARE>
__global__ void __launch_bounds__(64 * MAX_WAVES) talk_kernel(TalkArgs t) {
    extern __shared__ float s_dyn[];
    const AttnArgs &a = t.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = wave_id(), nw = blockDim.x >> 6, l16 = lane & 15, q4 = (lane >> 4) * 4, q8 = (lane >> 4) * 8;
    const int per_die = (t.items + 7) >> 3;
    const int id = t.many ? (int)(blockIdx.x & 7) * per_die + (int)(blockIdx.x >> 3) : (int)blockIdx.x;  // neighbours share keys: on one die
    if (id >= t.items) return;
    const int piece = id % a.pieces;
    int seq = id / a.pieces, ti = 0, count;
    if (t.many) {
        if (!item_of_seq(a.cu, a.n_seqs, 1 << t.lr, a.min_rows, id / a.pieces, &seq, &ti, &count)) return;
    } else if (!a.one_token && a.cu[seq + 1] - a.cu[seq] != 1) {
        return;
    }
    const int row0 = a.one_token ? seq : a.cu[seq] + (ti << t.lr), ntok = a.one_token ? 1 : min(1 << t.lr, a.cu[seq + 1] - row0);
    const int pos0 = a.pos[row0], pos_hi = pos0 + ntok - 1, last_blk = pos_hi / BS;
    const int g_first = first_key(a.p, pos0) / 32 + piece * (a.piece / 32), g_end = min(pos_hi / 32 + 1, g_first + a.piece / 32);
    const int all_from = first_key(a.p, pos_hi);
    const int vds = (a.p.v_dim + 3) / 4 * 4 + 4;  // floats of a partial result: the output, then maximum and sum
    const auto partial = [&](int row, int h) { return a.partial + (((size_t)(t.many ? row : seq) * a.p.heads + h) * a.pieces + piece) * vds; };
    if (g_first >= g_end) {  // nothing of this piece is seen
        for (int i = tid; i < ntok * a.p.heads; i += blockDim.x) {
            float *dst = partial(row0 + i / a.p.heads, i % a.p.heads) + vds - 4;
            dst[0] = -INFINITY, dst[1] = 0.f;
        }
        return;
    }
    const int tc = talk_cols(a.p.heads), m_tiles = (a.p.heads + 15) / 16, k_steps = (a.p.heads + 31) / 32;
    bf16 *s_talk = (bf16 *)(s_dyn + 2 * t.buf);
    for (int i = tid; i < m_tiles * 16 * tc; i += blockDim.x) {
        const int h = i / tc, g = i % tc;
        s_talk[i] = h < a.p.heads && g < a.p.heads ? ((const bf16 *)a.p.talk)[h * a.p.heads + g] : (bf16)0.f;
    }
    for (int i = tid; i < 2 * t.buf; i += blockDim.x) s_dyn[i] = 0.f;  // (heads that pad a row stay zero)
    __syncthreads();

    // this wave's tiles
    const int first_tile = wave * TPW, wave_tiles = min(TPW, t.tiles - first_tile);  // none or fewer for the last waves
    constexpr bool KEEP_Q = TPW <= 2;  // (four tiles: queries are read again for every group)
    Queries<KD, VD, TPW> qs;
    qs.clear();
    int tok[TPW], head[TPW], from[TPW], to[TPW][4];  // query lane % 16: its row, head, scores; pairs 4 (lane / 16) ..: where scores go
    const bf16 *qp[TPW];
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const int ti_ = min(first_tile + i, t.tiles - 1), g = ti_ / t.per_kv, sub = ti_ % t.per_kv, pairs = a.group << t.lr;
        const int m = min(sub * 16 + l16, pairs - 1), tt = min(m / a.group, ntok - 1);
        tok[i] = sub * 16 + l16 < pairs ? m / a.group : ntok, head[i] = g * a.group + m % a.group;
        from[i] = m / a.group * t.hs + head[i];
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int w = sub * 16 + q4 + r;
            to[i][r] = w < pairs ? w / a.group * t.hs + g * a.group + w % a.group : -1;
        }
        qs.pos[i] = pos0 + tt;
        qs.lo[i] = first_key(a.p, pos0 + tt);
        qs.lut[i] = 0;
        qs.qs[i] = score_factor(a.p, qs.pos[i]);
        qs.far[i] = score_offset(a.p, head[i]);
        qp[i] = (const bf16 *)a.p.q + (size_t)(row0 + tt) * a.p.ldq + head[i] * a.p.k_dim;
        if constexpr (KEEP_Q) {
#pragma unroll
            for (int kk = 0; kk < KD; kk++) qs.q[i][kk] = load_q(qp[i], kk * 32 + q8, a.p.k_dim, a.vec_q);
        }
    }
    const int32_t *bt = a.tables + (size_t)a.rows[seq] * a.max_blocks;
    const int g0 = min(first_tile, t.tiles - 1) / t.per_kv;
    Keys<KD, VD, 1, false> ks;
    ks.init(a, g0, lane);
    int b0 = bt[min(2 * g_first, last_blk)], b1 = bt[min(2 * g_first + 1, last_blk)];
    if (wave_tiles > 0) ks.load_k(b0, b1);
    const int pair_tiles = 2 << t.lr, row_mask = (1 << t.lr) - 1;
    for (int gi = g_first; gi < g_end; gi++) {
        float *buf = s_dyn + ((gi - g_first) & 1) * t.buf;
        const int k0 = gi * 32;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            if (i >= wave_tiles) break;
            if (!SHARE && i > 0) {
                ks.init(a, (first_tile + i) / t.per_kv, lane);
                ks.load_k(b0, b1);
            }
            f32x4 st[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int kk = 0; kk < KD; kk++) {
                const bf16x8 q = KEEP_Q ? qs.q[i][kk] : load_q(qp[i], kk * 32 + q8, a.p.k_dim, a.vec_q);
                st[0] = mma(q, ks.k[0][0][kk], st[0]);
                st[1] = mma(q, ks.k[0][1][kk], st[1]);
            }
#pragma unroll
            for (int h = 0; h < 2; h++) {  // column lane % 16 of tile h: this key
                float *dst = buf + key_at(t, (l16 >> 2) * 8 + h * 4 + (l16 & 3));
                if (t.vec) {
                    if (to[i][0] >= 0) *(f32x4 *)(dst + to[i][0]) = st[h];
                } else {
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (to[i][r] >= 0) dst[to[i][r]] = st[h][r];
                }
            }
        }
        const int v0 = b0, v1 = b1;
        if (SHARE && wave_tiles > 0) ks.load_v(v0, v1, lane);
        if (gi + 1 < g_end) {
            b0 = bt[min(2 * gi + 2, last_blk)], b1 = bt[min(2 * gi + 3, last_blk)];
            if (SHARE && wave_tiles > 0) ks.load_k(b0, b1);
        }
        __syncthreads();
        for (int nt = wave; nt < pair_tiles; nt += nw) {
            const int p = nt * 16 + l16;
            float *at = buf + key_at(t, p >> t.lr) + (p & row_mask) * t.hs;
            bf16x8 hi[2], lo[2];
#pragma unroll
            for (int k = 0; k < 2; k++) {
                const int g = k * 32 + q8;
                f32x4 x0 = f32x4{0.f, 0.f, 0.f, 0.f}, x1 = x0;
                if (g < t.h8) x0 = *(const f32x4 *)(at + g), x1 = *(const f32x4 *)(at + g + 4);
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const float v = e < 4 ? x0[e & 3] : x1[e & 3];
                    hi[k][e] = (bf16)v;
                    lo[k][e] = (bf16)(v - (float)hi[k][e]);
                }
            }
            for (int m = 0; m < m_tiles; m++) {
                f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int k = 0; k < 2; k++) {
                    if (k >= k_steps) break;
                    const bf16x8 w = *(const bf16x8 *)(s_talk + (m * 16 + l16) * tc + k * 32 + q8);
                    acc = mma(w, lo[k], acc);
                    acc = mma(w, hi[k], acc);
                }
                if (m * 16 + q4 < t.h8) *(f32x4 *)(at + m * 16 + q4) = acc;
            }
        }
        __syncthreads();
        const bool whole = k0 + 31 <= pos0 && k0 >= all_from;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            if (i >= wave_tiles) break;
            if (!SHARE) {
                ks.init(a, (first_tile + i) / t.per_kv, lane);
                ks.load_v(v0, v1, lane);
            }
            f32x4 st[2];
#pragma unroll
            for (int j = 0; j < 8; j++) st[j >> 2][j & 3] = buf[key_at(t, q8 + j) + from[i]];
            qs.template step<1, false>(a, ks, st[0], st[1], i, k0, lane, whole, true, nullptr);
        }
        if (!SHARE && gi + 1 < g_end && wave_tiles > 0) {
            ks.init(a, g0, lane);
            ks.load_k(b0, b1);
        }
    }
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        if (i >= wave_tiles) break;
        float l = qs.l[i];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        if (tok[i] >= ntok) continue;
        if (a.partial) {
            float *dst = partial(row0 + tok[i], head[i]);
            if (q4 == 0) dst[vds - 4] = qs.m[i], dst[vds - 3] = l;
#pragma unroll
            for (int v = 0; v < VD; v++)
                if (v * 16 + q4 < vds - 4) *(f32x4 *)(dst + v * 16 + q4) = qs.o[i][v];
        } else {
            const float inv = 1.0f / (l + sink_term(a.p, head[i], qs.m[i]));
#pragma unroll
            for (int v = 0; v < VD; v++) write4(a, row0 + tok[i], head[i], v * 16 + q4, qs.o[i][v] * inv);
        }
    }
}

// Pieces -> results: a wave per (row, head).
__global__ void __launch_bounds__(256) talk_merge_kernel(TalkArgs t) {
    const AttnArgs &a = t.a;
    const int h = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, vd = a.p.v_dim, vds = (vd + 3) / 4 * 4 + 4;
    if (h >= a.p.heads) return;
    int row = blockIdx.y;
    if (t.many) {
        const int seq = seq_of_row(a.cu, a.n_seqs, row);
        if (a.cu[seq + 1] - a.cu[seq] < a.min_rows) return;
    } else if (!a.one_token) {
        const int seq = row;
        row = a.cu[seq];
        if (a.cu[seq + 1] - row != 1) return;
    }
    const float *src = a.partial + ((size_t)blockIdx.y * a.p.heads + h) * a.pieces * vds;
    float m = -INFINITY, l = 0.f;
    for (int i = 0; i < a.pieces; i++) m = fmaxf(m, src[(size_t)i * vds + vds - 4]);
    for (int i = 0; i < a.pieces; i++) l += src[(size_t)i * vds + vds - 3] * __builtin_amdgcn_exp2f(src[(size_t)i * vds + vds - 4] - m);
    const float inv = a.p.out_scale / (l + sink_term(a.p, h, m));
    bf16 *out = (bf16 *)a.p.out + (size_t)row * a.p.ldo + h * vd;
    for (int d = lane; d < vd; d += 64) {
        float o = 0.f;
        for (int i = 0; i < a.pieces; i++) {
            const float f = __builtin_amdgcn_exp2f(src[(size_t)i * vds + vds - 4] - m);
            if (f > 0.f) o = fmaf(src[(size_t)i * vds + d], f, o);  // (what a piece that nobody saw holds is not read)
        }
        if (a.p.gate) o *= sigmoid_f((float)((const bf16 *)a.p.gate)[(size_t)row * a.p.ldg + h * vd + d]);
        out[d] = (bf16)(o * inv);
    }
}

// Fills in what follows from the rows of a workgroup; false when they do not fit.
bool plan(TalkArgs *t, int lr, int tpw) {
    t->lr = lr;
    t->per_kv = ceil_div(t->a.group << lr, 16);
    t->tiles = t->per_kv * t->a.p.kv_heads;
    t->h8 = (t->a.p.heads + 7) / 8 * 8, t->hs = t->h8 + 4;
    t->buf = (32 << lr) * t->hs + 64;
    t->vec = t->a.group % 4 == 0;
    return t->tiles <= MAX_WAVES * tpw && 2 * t->buf * 4 + (t->a.p.heads + 15) / 16 * 16 * talk_cols(t->a.p.heads) * 2 <= LDS_BYTES;
}

template <int KD, int VD, int TPW, bool SHARE>
void launch_as(vx_backend *be, const TalkArgs &t) {
    const size_t lds = 2 * (size_t)t.buf * 4 + (size_t)((t.a.p.heads + 15) / 16 * 16) * talk_cols(t.a.p.heads) * 2;
    static bool allowed = false;
    if (!allowed) {
        (void)hipFuncSetAttribute((const void *)talk_kernel<KD, VD, TPW, SHARE>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS_BYTES);
        allowed = true;
    }
    const int waves = std::max(4, ceil_div(t.tiles, TPW));
    talk_kernel<KD, VD, TPW, SHARE><<<t.many ? ceil_div(t.items, 8) * 8 : t.items, 64 * waves, lds, be->stream>>>(t);
}

template <int KD, int VD>
int launch(vx_backend *be, TalkArgs t, int tpw, int units, int rows) {
    t.items = units * t.a.pieces;
    t.a.partial = nullptr;
    if (t.a.pieces > 1) {
        const size_t bytes = (size_t)rows * t.a.p.heads * t.a.pieces * ((t.a.p.v_dim + 3) / 4 * 4 + 4) * 4;
        const int rc = ensure_ws(be, &be->attn_ws, &be->attn_ws_bytes, bytes, "attention");
        if (rc) return rc;
        t.a.partial = (float *)be->attn_ws;
        be->split.batch = 0;  // (whatever an earlier call left there is gone)
    }
    const bool share = t.per_kv % tpw == 0;
    if (tpw == 1)
        launch_as<KD, VD, 1, true>(be, t);
    else if (tpw == 2 && share)
        launch_as<KD, VD, 2, true>(be, t);
    else if (tpw == 2)
        launch_as<KD, VD, 2, false>(be, t);
    else
        launch_as<KD, VD, 4, false>(be, t);
    VX_CHECK_LAUNCH();
    if (t.a.pieces > 1) {
        talk_merge_kernel<<<dim3(ceil_div(t.a.p.heads, 4), rows), 256, 0, be->stream>>>(t);
        VX_CHECK_LAUNCH();
    }
    return VX_OK;
}

int launch(vx_backend *be, const TalkArgs &t, int tpw, int units, int rows) {
    const int wide = std::max(t.a.p.k_dim, t.a.p.v_dim);
    if (wide <= 64) return launch<2, 4>(be, t, tpw, units, rows);
    if (wide <= 96) return launch<3, 6>(be, t, tpw, units, rows);
    return launch<4, 8>(be, t, tpw, units, rows);
}

// The smallest number of tiles to a wave with which a workgroup takes one row.
int least_tpw(TalkArgs t) {
    for (int tpw = 1; tpw <= MAX_TPW; tpw *= 2)
        if (plan(&t, 0, tpw)) return tpw;
    return 0;
}

}  // namespace

namespace vx {

int attn_talk(vx_backend *be, AttnArgs a, const vx_ragged *b) {
    TalkArgs t;
    memset(&t, 0, sizeof t);
    t.a = a;
    t.a.min_rows = std::max(a.p.min_rows, 2);
    bool any_one = !b->q_lens && a.p.min_rows <= 1;
    int64_t many = 0;
    if (b->q_lens)
        for (int s = 0; s < b->n_seqs; s++) {
            any_one |= b->q_lens[s] == 1 && a.p.min_rows <= 1;
            if (b->q_lens[s] >= t.a.min_rows) many += b->q_lens[s];
        }
    // keys of `rows` neighbouring rows, from the start of their first group of 32 on
    const auto span = [&](int rows) {
        int64_t n = b->max_kv_len;
        if (a.p.window > 0) n = std::min<int64_t>(n, (int64_t)a.p.window + rows - 1 + 31);
        if (a.p.chunk > 0) n = std::min<int64_t>(n, (int64_t)a.p.chunk + rows - 1 + 31);
        return (int)n;
    };
    if (many > 0) {
        t.many = 1;
        // rows that share a wave's keys: as many as two tiles a wave hold
        int tpw = std::max(2, least_tpw(t)), lr = 0;
        while ((2 << lr) <= MAX_ROWS && plan(&t, lr + 1, tpw)) lr++;
        plan(&t, lr, tpw);
        if (t.tiles <= MAX_WAVES) tpw = 1;
        const int units = count_items(b, 1 << lr, t.a.min_rows), n = span(1 << lr);
        const int want = units >= 256 ? 1 : ceil_div(512, units);
        t.a.piece = std::max(128, ceil_div(ceil_div(n, want), 32) * 32);
        t.a.pieces = ceil_div(n, t.a.piece);
        const int rc = launch(be, t, tpw, units, b->rows);
        if (rc) return rc;
    }
    if (any_one) {
        t.many = 0;
        const int tpw = least_tpw(t);
        plan(&t, 0, tpw);
        const int n = span(1);
        t.a.piece = (int64_t)b->n_seqs * ceil_div(n, 256) < 512 ? 128 : 256;
        t.a.pieces = ceil_div(n, t.a.piece);
        const int rc = launch(be, t, tpw, b->n_seqs, b->n_seqs);
        if (rc) return rc;
    }
    return VX_OK;
}

}  // namespace vx

extern "C" int vx_attn_talk_fast(int act, int block_size, int heads, int kv_heads, int k_dim, int v_dim) {
    if (heads < 1 || heads > MAX_HEADS || kv_heads < 1 || heads % kv_heads || k_dim < 1 || v_dim < 1) return 0;
    if (act != VX_ACT_BF16 || block_size != BS || std::max(k_dim, v_dim) > 128) return 0;
    TalkArgs t;
    memset(&t, 0, sizeof t);
    t.a.p.heads = heads, t.a.p.kv_heads = kv_heads, t.a.p.k_dim = k_dim, t.a.p.v_dim = v_dim, t.a.group = heads / kv_heads;
    return least_tpw(t) > 0;
}
