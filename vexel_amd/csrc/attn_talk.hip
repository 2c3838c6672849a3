// Paged attention whose scores are mixed across heads ahead of the softmax (vx_attn_ragged with talk), on the bfloat16 matrix cores.
//
// A workgroup takes a few rows of one sequence with all heads, and walks a piece of their keys in groups of 32. A wave owns up to four
// tiles of 16 (row, head) pairs of one K/V head each. A group takes three stages:
//   scores   every wave's products Q K^T to LDS, float32 [key][row][head]
//   mix      talk * scores over 16 (key, row) pairs at a time, in place; the scores enter the product as two bfloat16 parts
//   output   every wave reads its tiles' mixed scores back, a lane eight consecutive keys of one query, for softmax and O^T = V^T P^T
// Two buffers of scores take turns: a group is mixed while the next one's scores are made, and two barriers a group are enough. Pieces of
// keys: partial results that a second launch merges.
#include <string.h>

#include <algorithm>

#include "attn_tiles.h"

using namespace vx;

namespace {

constexpr int MAX_WAVES = 8, MAX_TPW = 4, MAX_ROWS = 32, MAX_HEADS = 64;
constexpr int LDS_BYTES = 156 * 1024;

struct TalkArgs {
    AttnArgs a;
    int lr;               // log2 of the rows of a workgroup
    int per_kv, tiles;    // tiles of a K/V head; of all
    int hs, h8;           // floats from one row's scores to the next; heads up to a multiple of 8
    int buf;              // floats of a buffer
    int many;             // sequences with several rows (else those with one)
    int items;            // (row tile, piece) pairs
};

__host__ __device__ __forceinline__ int talk_cols(int heads) { return (heads + 31) / 32 * 32 + 8; }  // LDS row of the talk matrix

constexpr bool queries_in_lds(int kd, int tpw, bool share) { return kd == 4 && tpw == 2 && share; }

// Where the score of a key (0 .. 31 of the group) lies; head and row are added.
__device__ __forceinline__ int key_at(const TalkArgs &t, int key) { return (key << t.lr) * t.hs + (key >> 3) * 16; }

// VEC: four pairs of a lane are neighbouring heads of one row.
template <int KD, int VD, int TPW, bool SHARE, bool VEC>
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
    // this wave's tiles
    const int first_tile = wave * TPW, wave_tiles = min(TPW, t.tiles - first_tile);  // none or fewer for the last waves
    const int32_t *bt = a.tables + (size_t)a.rows[seq] * a.max_blocks;
    Keys<KD, VD, 1, false> ks;
    ks.init(a, min(first_tile, t.tiles - 1) / t.per_kv, lane);
    const auto block = [&](int b) { return bt[min(b, last_blk)]; };
    int b0 = block(2 * g_first), b1 = block(2 * g_first + 1), n0 = block(2 * g_first + 2), n1 = block(2 * g_first + 3);
    int f0 = block(2 * g_first + 4), f1 = block(2 * g_first + 5);  // (read from the table a group before their keys are)
    if (SHARE && wave_tiles > 0) ks.load_k(b0, b1);
    // queries: in registers, in LDS where registers are short, or (four tiles) read again for every group
    constexpr bool LDS_Q = queries_in_lds(KD, TPW, SHARE), KEEP_Q = TPW <= 2 && !LDS_Q;
    bf16x8 *s_q = (bf16x8 *)(s_talk + m_tiles * 16 * tc) + wave * TPW * KD * 64 + lane;
    Queries<KD, VD, TPW> qs;
    qs.clear();
    int from[TPW], to[TPW][VEC ? 1 : 4];  // query lane % 16: its scores; pairs 4 (lane / 16) ..: where scores go (-1: nowhere)
    const bf16 *qp[TPW];
    const int pairs = a.group << t.lr;
    const auto tile_of = [&](int i) { return min(first_tile + i, t.tiles - 1); };
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const int g = tile_of(i) / t.per_kv, sub = tile_of(i) % t.per_kv;
        const int m = min(sub * 16 + l16, pairs - 1), tt = min(m / a.group, ntok - 1), h = g * a.group + m % a.group;
        from[i] = m / a.group * t.hs + h;
#pragma unroll
        for (int r = 0; r < (VEC ? 1 : 4); r++) {
            const int w = sub * 16 + q4 + r;
            to[i][r] = w < pairs ? w / a.group * t.hs + g * a.group + w % a.group : -1;
        }
        qs.pos[i] = pos0 + tt;
        qs.lo[i] = first_key(a.p, pos0 + tt);
        qs.lut[i] = 0;
        qs.qs[i] = score_factor(a.p, qs.pos[i]);
        qs.far[i] = score_offset(a.p, h);
        qp[i] = (const bf16 *)a.p.q + (size_t)(row0 + tt) * a.p.ldq + h * a.p.k_dim;
#pragma unroll
        for (int kk = 0; kk < KD; kk++) {
            if constexpr (KEEP_Q) qs.q[i][kk] = load_q(qp[i], kk * 32 + q8, a.p.k_dim, a.vec_q);
            if constexpr (LDS_Q) s_q[(i * KD + kk) * 64] = load_q(qp[i], kk * 32 + q8, a.p.k_dim, a.vec_q);  // (this wave alone reads it)
        }
    }
    // this wave's products with the keys of a group to a buffer; the keys of tiles that share them are there already
    const int my_key = (l16 >> 2) * 8 + (l16 & 3);  // of the first 16 columns; of the others it is four further on
    const auto scores = [&](float *buf, int b0, int b1) {
        float *dst = buf + key_at(t, my_key);
        const int next_half = key_at(t, my_key + 4) - key_at(t, my_key);
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            if (i >= wave_tiles) break;
            if constexpr (!SHARE) {
                ks.init(a, tile_of(i) / t.per_kv, lane);
                ks.load_k(b0, b1);
            }
            f32x4 st[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int kk = 0; kk < KD; kk++) {
                const bf16x8 q = KEEP_Q ? qs.q[i][kk] : LDS_Q ? s_q[(i * KD + kk) * 64] : load_q(qp[i], kk * 32 + q8, a.p.k_dim, a.vec_q);
                st[0] = mma(q, ks.k[0][0][kk], st[0]);
                st[1] = mma(q, ks.k[0][1][kk], st[1]);
            }
#pragma unroll
            for (int h = 0; h < 2; h++) {
                if constexpr (VEC) {
                    if (to[i][0] >= 0) *(f32x4 *)(dst + h * next_half + to[i][0]) = st[h];
                } else {
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (to[i][r] >= 0) dst[h * next_half + to[i][r]] = st[h][r];
                }
            }
        }
    };
    const int pair_tiles = 2 << t.lr, row_mask = (1 << t.lr) - 1;
    // two operands at a time: of two tiles of pairs, or (more than 32 heads) the two of one tile
    const bool deep = k_steps > 1;
    const auto mix = [&](float *buf) {
        for (int nt = wave; nt < pair_tiles; nt += deep ? nw : 2 * nw) {
            const bool both = deep || nt + nw < pair_tiles;
            float *at[2];
            bf16x8 hi[2], lo[2];
#pragma unroll
            for (int u = 0; u < 2; u++) {
                if (u > 0 && !both) break;
                const int p = (nt + (deep ? 0 : u * nw)) * 16 + l16, g = (deep ? u * 32 : 0) + q8;
                at[u] = buf + key_at(t, p >> t.lr) + (p & row_mask) * t.hs;
                f32x4 x0 = f32x4{0.f, 0.f, 0.f, 0.f}, x1 = x0;
                if (g < t.h8) x0 = *(const f32x4 *)(at[u] + g), x1 = *(const f32x4 *)(at[u] + g + 4);
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const float v = e < 4 ? x0[e & 3] : x1[e & 3];
                    hi[u][e] = (bf16)v;
                    lo[u][e] = (bf16)(v - (float)hi[u][e]);
                }
            }
            for (int m = 0; m < m_tiles; m++) {
                const bf16 *row = s_talk + (m * 16 + l16) * tc + q8;
                bf16x8 w = *(const bf16x8 *)row;
                f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f}, more = acc;
                acc = mma(w, lo[0], acc);
                acc = mma(w, hi[0], acc);
                if (both) {
                    if (deep) w = *(const bf16x8 *)(row + 32);
                    more = mma(w, lo[1], more);
                    more = mma(w, hi[1], more);
                }
                if (m * 16 + q4 < t.h8) {
                    *(f32x4 *)(at[0] + m * 16 + q4) = deep ? acc + more : acc;
                    if (both && !deep) *(f32x4 *)(at[1] + m * 16 + q4) = more;
                }
            }
        }
    };
    for (int i = tid; i < m_tiles * 16 * tc; i += blockDim.x) {
        const int h = i / tc, g = i % tc;
        s_talk[i] = h < a.p.heads && g < a.p.heads ? ((const bf16 *)a.p.talk)[h * a.p.heads + g] : (bf16)0.f;
    }
    if (t.h8 > a.p.heads)
        for (int i = tid; i < 2 * t.buf; i += blockDim.x) s_dyn[i] = 0.f;  // (heads that pad a row stay zero)
    __syncthreads();
    if (wave_tiles > 0) {
        scores(s_dyn, b0, b1);
        if (SHARE) ks.load_k(n0, n1);  // (behind the last group: its own last block again)
    }
    for (int gi = g_first; gi < g_end; gi++) {
        float *buf = s_dyn + ((gi - g_first) & 1) * t.buf, *other = s_dyn + ((gi - g_first + 1) & 1) * t.buf;
        const int k0 = gi * 32;
        const int e0 = block(2 * gi + 6), e1 = block(2 * gi + 7);
        __syncthreads();
        mix(buf);
        if (gi + 1 < g_end && wave_tiles > 0) scores(other, n0, n1);  // (that buffer's scores were read before the barrier)
        if (SHARE && wave_tiles > 0) ks.load_v(b0, b1, lane), ks.load_k(f0, f1);
        __syncthreads();
        const bool whole = k0 + 31 <= pos0 && k0 >= all_from;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            if (i >= wave_tiles) break;
            if constexpr (!SHARE) {
                ks.init(a, tile_of(i) / t.per_kv, lane);
                ks.load_v(b0, b1, lane);
            }
            f32x4 st[2];
#pragma unroll
            for (int j = 0; j < 8; j++) st[j >> 2][j & 3] = buf[key_at(t, q8 + j) + from[i]];
            qs.template step<1, false>(a, ks, st[0], st[1], i, k0, lane, whole, true, nullptr);
        }
        b0 = n0, b1 = n1, n0 = f0, n1 = f1, f0 = e0, f1 = e1;
    }
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        if (i >= wave_tiles) break;
        float l = qs.l[i];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        const int g = tile_of(i) / t.per_kv, m = tile_of(i) % t.per_kv * 16 + l16, tok = m / a.group, head = g * a.group + m % a.group;
        if (m >= pairs || tok >= ntok) continue;
        if (a.partial) {
            float *dst = partial(row0 + tok, head);
            if (q4 == 0) dst[vds - 4] = qs.m[i], dst[vds - 3] = l;
#pragma unroll
            for (int v = 0; v < VD; v++)
                if (v * 16 + q4 < vds - 4) *(f32x4 *)(dst + v * 16 + q4) = qs.o[i][v];
        } else {
            const float inv = 1.0f / (l + sink_term(a.p, head, qs.m[i]));
#pragma unroll
            for (int v = 0; v < VD; v++) write4(a, row0 + tok, head, v * 16 + q4, qs.o[i][v] * inv);
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
    // a lane looks after a piece (every 64th)
    float m = -INFINITY, l = 0.f;
    for (int i = lane; i < a.pieces; i += 64) m = fmaxf(m, src[(size_t)i * vds + vds - 4]);
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
    float o[2] = {0.f, 0.f};  // columns lane and lane + 64
    for (int first = 0; first < a.pieces; first += 64) {
        int n = min(64, a.pieces - first);
        float f = 0.f;
        if (lane < n) {
            const float *ml = src + (size_t)(first + lane) * vds + vds - 4;
            f = __builtin_amdgcn_exp2f(ml[0] - m);
            l = fmaf(ml[1], f, l);
        }
        const uint64_t seen = __ballot(f > 0.f);
        n = seen ? 64 - __builtin_clzll(seen) : 0;  // (the last pieces of early rows are empty)
        for (int i = 0; i < n; i += 4) {
            float w[4], v[4][2];
#pragma unroll
            for (int u = 0; u < 4; u++) {
                w[u] = __shfl(f, min(i + u, 63), 64);  // (0 beyond the last)
                const float *row = src + (size_t)(first + min(i + u, n - 1)) * vds;
#pragma unroll
                for (int x = 0; x < 2; x++) v[u][x] = row[min(lane + x * 64, vd - 1)];
            }
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int x = 0; x < 2; x++) o[x] = fmaf(w[u] > 0.f ? v[u][x] : 0.f, w[u], o[x]);  // (what a piece that nobody saw holds does not count)
        }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) l += __shfl_xor(l, off, 64);
    const float inv = a.p.out_scale / (l + sink_term(a.p, h, m));
    bf16 *out = (bf16 *)a.p.out + (size_t)row * a.p.ldo + h * vd;
#pragma unroll
    for (int x = 0; x < 2; x++)
        if (const int d = lane + x * 64; d < vd) {
            const float gate = a.p.gate ? sigmoid_f((float)((const bf16 *)a.p.gate)[(size_t)row * a.p.ldg + h * vd + d]) : 1.0f;
            out[d] = (bf16)(o[x] * gate * inv);
        }
}

int wide_of(const TalkArgs &t) { return std::max(t.a.p.k_dim, t.a.p.v_dim); }
int kd_of(const TalkArgs &t) { return wide_of(t) <= 64 ? 2 : wide_of(t) <= 96 ? 3 : 4; }
int waves_of(const TalkArgs &t, int tpw) { return std::max(4, ceil_div(t.tiles, tpw)); }

size_t lds_bytes(const TalkArgs &t, int tpw) {
    const size_t q = queries_in_lds(kd_of(t), tpw, t.per_kv % tpw == 0) ? (size_t)waves_of(t, tpw) * tpw * kd_of(t) * 1024 : 0;
    return 2 * (size_t)t.buf * 4 + (size_t)((t.a.p.heads + 15) / 16 * 16) * talk_cols(t.a.p.heads) * 2 + q;
}

// Fills in what follows from the rows of a workgroup; false when they do not fit.
bool plan(TalkArgs *t, int lr, int tpw) {
    t->lr = lr;
    t->per_kv = ceil_div(t->a.group << lr, 16);
    t->tiles = t->per_kv * t->a.p.kv_heads;
    t->h8 = (t->a.p.heads + 7) / 8 * 8, t->hs = t->h8 + 4;
    t->buf = (32 << lr) * t->hs + 64;
    return t->tiles <= MAX_WAVES * tpw && lds_bytes(*t, tpw) <= LDS_BYTES;
}

template <int KD, int VD, int TPW, bool SHARE, bool VEC>
void launch_as(vx_backend *be, const TalkArgs &t) {
    const size_t lds = lds_bytes(t, TPW);
    static bool allowed = false;
    if (!allowed) {
        (void)hipFuncSetAttribute((const void *)talk_kernel<KD, VD, TPW, SHARE, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS_BYTES);
        allowed = true;
    }
    talk_kernel<KD, VD, TPW, SHARE, VEC><<<t.many ? ceil_div(t.items, 8) * 8 : t.items, 64 * waves_of(t, TPW), lds, be->stream>>>(t);
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
    const bool share = t.per_kv % tpw == 0, vec = t.a.group % 4 == 0;
    if (tpw == 1)
        vec ? launch_as<KD, VD, 1, true, true>(be, t) : launch_as<KD, VD, 1, true, false>(be, t);
    else if (tpw == 2 && share)
        vec ? launch_as<KD, VD, 2, true, true>(be, t) : launch_as<KD, VD, 2, true, false>(be, t);
    else if (tpw == 2)
        vec ? launch_as<KD, VD, 2, false, true>(be, t) : launch_as<KD, VD, 2, false, false>(be, t);
    else
        launch_as<KD, VD, 4, false, false>(be, t);
    VX_CHECK_LAUNCH();
    if (t.a.pieces > 1) {
        talk_merge_kernel<<<dim3(ceil_div(t.a.p.heads, 4), rows), 256, 0, be->stream>>>(t);
        VX_CHECK_LAUNCH();
    }
    return VX_OK;
}

int launch(vx_backend *be, const TalkArgs &t, int tpw, int units, int rows) {
    if (kd_of(t) == 2) return launch<2, 4>(be, t, tpw, units, rows);
    if (kd_of(t) == 3) return launch<3, 6>(be, t, tpw, units, rows);
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
        // (fewer where that leaves much of the chip without work)
        while (lr > 0 && t.tiles > MAX_WAVES && count_items(b, 1 << lr, t.a.min_rows) < 64) plan(&t, --lr, tpw);
        if (t.tiles <= MAX_WAVES) tpw = 1;
        const int units = count_items(b, 1 << lr, t.a.min_rows), n = span(1 << lr);
        const int want = units >= 192 ? 1 : ceil_div(256, units);  // (a workgroup fills a compute unit)
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
