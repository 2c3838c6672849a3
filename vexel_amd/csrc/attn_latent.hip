// Latent attention for mixed batches: what a token leaves in the paged pool (vx_latent_store), causal attention over it
// (vx_attn_latent), and the spreading of the rotated key part for layers that spell their keys out (vx_latent_spread).
//
// A pool row is one token: c [pad] | rotated key part [64 or more]. All heads read the same rows, so a workgroup takes
// 16, 32 or 64 (row, head) pairs of one sequence through a piece of its keys, a tile of keys at a time:
//   tile -> LDS (each wave brings a quarter of it, requested a tile ahead into registers)
//   S^T = K Q^T       waves split the tile's keys and the queries; the queries' operands stay in registers
//   running maximum   exchanged through LDS, the weights go to LDS as two bfloat16 parts (16 bits of the 24)
//   O^T += V^T P^T    V is the first part of the same rows, read transposed (ds_read_tr); waves split the dimensions
// Pieces leave partial results that a second launch merges, which also counts the sink.
#include <string.h>

#include "attn_plain.h"

using namespace vx;

namespace {

constexpr int BS = 16;  // tokens of a block (matrix-core kernel)

struct Args {
    vx_latent_attn_args p;
    const int32_t *cu, *pos, *rows, *kv_lens, *tables;
    int n_seqs, max_blocks, one_token;
    int decode;               // items are the sequences that bring one row; otherwise tiles of the others
    int min_rows, max_rows, tiles, per_tile;
    int piece, pieces, n_rows;
    float *partial;           // [row][head][piece][pad], then the same of (maximum, sum)
};

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));

// Four rows x 16 columns of 16-bit elements, transposed on the way: of a group of 16 lanes, lane i points at columns 4 (i & 3) ..
// of row i >> 2 and gets column i of the four rows.
__device__ __forceinline__ s16x4 read_transposed(const void *p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4 *)p);
}

__device__ __forceinline__ float sink_term(const vx_latent_attn_args &p, int h, float m) {
    return p.sink ? __builtin_amdgcn_exp2f(p.sink[h] * kLog2e - m) : 0.f;
}

template <int RT, int MT>
__global__ void __launch_bounds__(256, MT == 1 ? 2 : 1) latent_kernel(Args a) {
    constexpr int CPR = RT * 8 + 8;                   // 16-byte pieces of a pool row
    constexpr int KT = MT == 1 ? 64 : 32;             // keys of a tile
    constexpr int WK = 4 / MT, NK = KT / 16 / WK;     // waves over keys; 16-key tiles of a wave
    constexpr int KR = KT / 4, LOADS = KR * CPR / 64; // rows and pieces that a wave brings
    constexpr int KK = RT * 2 + 2;                    // steps of 32 dimensions
    constexpr int PS = KT + 8;                        // a query's weights in LDS
    __shared__ u32x4 s_k[KT * CPR];                   // pieces of a row permuted within eight by the row's low bits
    __shared__ bf16 s_hi[MT * 16 * PS], s_lo[MT * 16 * PS];
    __shared__ float s_max[WK][MT * 16], s_l[WK][MT * 16];
    const vx_latent_attn_args &p = a.p;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, kw = wave % WK, mw = wave / WK, li = lane & 15, lq = lane >> 4;
    const int H = p.heads;
    int seq, m_first, piece, row0, n;
    if (a.decode) {
        piece = blockIdx.x, seq = blockIdx.y, m_first = blockIdx.z * MT * 16, n = 1;
        row0 = a.one_token ? seq : a.cu[seq];
        if (!a.one_token && a.cu[seq + 1] - row0 != 1) return;
    } else {
        int ti, count;
        if (!item_of_seq(a.cu, a.n_seqs, a.per_tile, a.min_rows, a.tiles - 1 - blockIdx.x, &seq, &ti, &count, H, a.max_rows)) return;
        piece = blockIdx.y, m_first = ti * MT * 16;
        row0 = a.cu[seq], n = a.cu[seq + 1] - row0;
    }
    const int pos0 = a.kv_lens[seq] - n, pairs = n * H;
    const int pos_hi = pos0 + min((m_first + MT * 16 - 1) / H, n - 1);
    const int k_lo = piece * a.piece, k_hi = min(pos_hi + 1, k_lo + a.piece);
    if (k_lo >= k_hi) return;
    const int32_t *bt = a.tables + (size_t)a.rows[seq] * a.max_blocks;
    const int last_blk = pos_hi / BS;

    // this wave's queries
    const int m_own = min(m_first + mw * 16 + li, pairs - 1), tok_own = m_own / H, head_own = m_own - tok_own * H;
    const int pos_own = pos0 + tok_own;
    bf16x8 qf[KK];
    {
        const bf16 *q = (const bf16 *)p.q + (size_t)(row0 + tok_own) * p.ldq + (size_t)head_own * (RT * 64) + lq * 8;
        const bf16 *r = (const bf16 *)p.qr + (size_t)(row0 + tok_own) * p.ldqr + (size_t)head_own * p.qr_stride + lq * 8;
        const int rot16 = (p.rot_dim + 15) & ~15;
#pragma unroll
        for (int kk = 0; kk < RT * 2; kk++) qf[kk] = *(const bf16x8 *)(q + kk * 32);
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            if (kk * 32 + lq * 8 < rot16) {
                qf[RT * 2 + kk] = *(const bf16x8 *)(r + kk * 32);
            } else {
#pragma unroll
                for (int j = 0; j < 8; j++) qf[RT * 2 + kk][j] = (bf16)0.f;
            }
        }
    }
    const float qs = p.scale * kLog2e;
    float m[MT], mo = -INFINITY, l = 0.f;             // running maxima of all queries, of the own; the own share of the sum
    f32x4 o[MT][RT];
#pragma unroll
    for (int t = 0; t < MT; t++) {
        m[t] = -INFINITY;
#pragma unroll
        for (int v = 0; v < RT; v++) o[t][v] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    u32x4 pf[LOADS];
    const u32x4 *pool = (const u32x4 *)p.pool;
    auto fetch = [&](int k0) {                        // a quarter of the tile lies inside one block: one run of memory
        const int r0 = k0 + wave * KR, blk = bt[min(r0 / BS, last_blk)];
        const u32x4 *src = pool + ((size_t)blk * BS + r0 % BS) * CPR + lane;
#pragma unroll
        for (int i = 0; i < LOADS; i++) pf[i] = MT == 1 ? __builtin_nontemporal_load(src + i * 64) : src[i * 64];
    };
    fetch(k_lo);
    for (int k0 = k_lo; k0 < k_hi; k0 += KT) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int idx = lane + i * 64, r = wave * KR + idx / CPR, c = idx % CPR;
            s_k[r * CPR + ((c & ~7) | ((c ^ r) & 7))] = pf[i];
        }
        __syncthreads();
        if (k0 + KT < k_hi) fetch(k0 + KT);
        f32x4 s[NK];
        float mx = -INFINITY;
#pragma unroll
        for (int nk = 0; nk < NK; nk++) {
            const int r = (kw * NK + nk) * 16 + li;
            s[nk] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KK; kk++) {
                const int c = kk * 4 + lq;
                s[nk] = mma(*(const bf16x8 *)&s_k[r * CPR + ((c & ~7) | ((c ^ r) & 7))], qf[kk], s[nk]);
            }
            const int key = k0 + (kw * NK + nk) * 16 + lq * 4;
#pragma unroll
            for (int j = 0; j < 4; j++) {
                s[nk][j] = key + j <= pos_own ? s[nk][j] * qs : -INFINITY;
                mx = fmaxf(mx, s[nk][j]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        if (lane < 16) s_max[kw][mw * 16 + lane] = mx;
        __syncthreads();
        float al[MT];
        bool moved = false;
#pragma unroll
        for (int t = 0; t < MT; t++) {
            float mn = m[t];
#pragma unroll
            for (int w = 0; w < WK; w++) mn = fmaxf(mn, s_max[w][t * 16 + li]);
            al[t] = mn > -INFINITY ? __builtin_amdgcn_exp2f(m[t] - mn) : 1.0f;
            moved |= mn > m[t];
            m[t] = mn;
        }
        {
            float mn = mo;
#pragma unroll
            for (int w = 0; w < WK; w++) mn = fmaxf(mn, s_max[w][mw * 16 + li]);
            if (mn > -INFINITY) l *= __builtin_amdgcn_exp2f(mo - mn);
            mo = mn;
            const float ref = mn > -INFINITY ? mn : 0.f;
#pragma unroll
            for (int nk = 0; nk < NK; nk++) {
                bf16x4 hi, lo;
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    const float e = __builtin_amdgcn_exp2f(s[nk][j] - ref);
                    l += e;
                    hi[j] = (bf16)e;
                    lo[j] = (bf16)(e - (float)hi[j]);
                }
                const int at = (mw * 16 + li) * PS + (kw * NK + nk) * 16 + lq * 4;
                *(bf16x4 *)&s_hi[at] = hi;
                *(bf16x4 *)&s_lo[at] = lo;
            }
        }
        __syncthreads();
        if (__any(moved)) {
#pragma unroll
            for (int t = 0; t < MT; t++)
#pragma unroll
                for (int v = 0; v < RT; v++) o[t][v] *= al[t];
        }
#pragma unroll
        for (int ks = 0; ks < KT / 32; ks++) {
            bf16x8 hi[MT], lo[MT];
#pragma unroll
            for (int t = 0; t < MT; t++) {
                const int at = (t * 16 + li) * PS + ks * 32 + lq * 8;
                hi[t] = *(const bf16x8 *)&s_hi[at];
                lo[t] = *(const bf16x8 *)&s_lo[at];
            }
#pragma unroll
            for (int v = 0; v < RT; v++) {
                s16x8 vt;
#pragma unroll
                for (int half = 0; half < 2; half++) {
                    const int r = ks * 32 + lq * 8 + half * 4 + (li >> 2), c = (wave * RT + v) * 2 + ((li & 3) >> 1);
                    const s16x4 x = read_transposed((const char *)&s_k[r * CPR + ((c & ~7) | ((c ^ r) & 7))] + (li & 1) * 8);
#pragma unroll
                    for (int j = 0; j < 4; j++) vt[half * 4 + j] = x[j];
                }
                const bf16x8 vb = __builtin_bit_cast(bf16x8, vt);
#pragma unroll
                for (int t = 0; t < MT; t++) {
                    o[t][v] = mma(vb, hi[t], o[t][v]);
                    o[t][v] = mma(vb, lo[t], o[t][v]);
                }
            }
        }
        __syncthreads();  // (the tile and the weights are done with)
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (lane < 16) s_l[kw][mw * 16 + lane] = l;
    __syncthreads();
#pragma unroll
    for (int t = 0; t < MT; t++) {
        const int q = m_first + t * 16 + li;
        if (q >= pairs) continue;
        const int tok = q / H, head = q - tok * H;
        float sum = 0.f;
#pragma unroll
        for (int w = 0; w < WK; w++) sum += s_l[w][t * 16 + li];
        if (a.pieces == 1) {
            const float inv = 1.0f / (sum + sink_term(p, head, m[t]));
            bf16 *out = (bf16 *)p.out + (size_t)(row0 + tok) * p.ldo + (size_t)head * (RT * 64) + lq * 4;
#pragma unroll
            for (int v = 0; v < RT; v++) store4(out + (wave * RT + v) * 16, o[t][v] * inv);
        } else {
            const size_t at = ((size_t)(row0 + tok) * H + head) * a.pieces + piece;
            float *dst = a.partial + at * (RT * 64) + lq * 4;
#pragma unroll
            for (int v = 0; v < RT; v++) *(f32x4 *)(dst + (wave * RT + v) * 16) = o[t][v];
            if (wave == 0 && lq == 0) {
                float *ml = a.partial + (size_t)a.n_rows * H * a.pieces * (RT * 64) + at * 2;
                ml[0] = m[t], ml[1] = sum;
            }
        }
    }
}

// One (row, head): its pieces become one.
__global__ void __launch_bounds__(128) latent_merge_kernel(Args a, int pad) {
    const int h = blockIdx.x, row = blockIdx.y;
    const int seq = a.one_token ? row : seq_of_row(a.cu, a.n_seqs, row);
    const int brings = a.one_token ? 1 : a.cu[seq + 1] - a.cu[seq];
    if (a.decode ? brings != 1 : (brings < a.min_rows || (a.max_rows > 0 && brings > a.max_rows))) return;
    const int n = a.pos[row] / a.piece + 1;
    const size_t at = ((size_t)row * a.p.heads + h) * a.pieces;
    const float *src = a.partial + at * pad, *ml = a.partial + (size_t)a.n_rows * a.p.heads * a.pieces * pad + at * 2;
    float m = -INFINITY, l = 0.f;
    for (int i = 0; i < n; i++) m = fmaxf(m, ml[2 * i]);
    for (int i = 0; i < n; i++) l += ml[2 * i + 1] * __builtin_amdgcn_exp2f(ml[2 * i] - m);
    const float inv = 1.0f / (l + sink_term(a.p, h, m));
    for (int d = threadIdx.x * 4; d < pad; d += blockDim.x * 4) {
        f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int i = 0; i < n; i++) o += *(const f32x4 *)(src + (size_t)i * pad + d) * __builtin_amdgcn_exp2f(ml[2 * i] - m);
        store4((bf16 *)a.p.out + (size_t)row * a.p.ldo + (size_t)h * pad + d, o * inv);
    }
}

template <int RT>
void launch_latent(vx_backend *be, const Args &a, int mt, dim3 grid) {
    if (mt == 1)
        latent_kernel<RT, 1><<<grid, 256, 0, be->stream>>>(a);
    else if (mt == 2)
        latent_kernel<RT, 2><<<grid, 256, 0, be->stream>>>(a);
    else
        latent_kernel<RT, 4><<<grid, 256, 0, be->stream>>>(a);
}

// Query tiles of 16 a workgroup takes.
int query_tiles(int64_t pairs) { return pairs <= 16 ? 1 : pairs <= 32 ? 2 : 4; }

template <int RT>
int run_latent(vx_backend *be, Args a, const vx_ragged *b) {
    const int H = a.p.heads, pad = RT * 64;
    const int64_t most = (int64_t)1 << 30;  // bytes of partial results
    int64_t one = b->q_lens ? 0 : b->n_seqs, longest = 0;
    a.min_rows = 2, a.max_rows = a.p.max_rows;
    if (b->q_lens)
        for (int s = 0; s < b->n_seqs; s++) {
            one += b->q_lens[s] == 1;
            if (b->q_lens[s] > 1 && (a.max_rows <= 0 || b->q_lens[s] <= a.max_rows) && b->q_lens[s] > longest) longest = b->q_lens[s];
        }
    a.n_rows = b->rows;
    const auto split = [&](int64_t wgs, int least) -> int {  // pieces, so that the launch fills the chip
        int64_t piece = 1024;
        while (piece > least && wgs * ceil_div(b->max_kv_len, (int)piece) < 512) piece /= 2;
        while ((int64_t)b->rows * H * ceil_div(b->max_kv_len, (int)piece) * (pad + 2) * 4 > most && piece < b->max_kv_len) piece *= 2;
        if (wgs >= 512) piece = b->max_kv_len;
        a.piece = ceil_div((int)piece, 64) * 64;
        a.pieces = ceil_div(b->max_kv_len, a.piece);
        if (a.pieces == 1) return VX_OK;
        const size_t bytes = (size_t)b->rows * H * a.pieces * (pad + 2) * 4;
        const int rc = ensure_ws(be, &be->attn_ws, &be->attn_ws_bytes, bytes, "attention");
        a.partial = (float *)be->attn_ws;
        be->split.batch = 0;  // (whatever an earlier call left there is gone)
        return rc;
    };
    const auto merge = [&]() {
        if (a.pieces > 1)
            latent_merge_kernel<<<dim3(H, b->rows), pad / 4 < 64 ? 64 : 128, 0, be->stream>>>(a, pad);
    };
    if (longest > 0) {
        const int mt = query_tiles(longest * H);
        a.decode = 0, a.per_tile = mt * 16;
        int64_t tiles = 0;
        for (int s = 0; s < b->n_seqs; s++)
            if (b->q_lens[s] > 1 && (a.max_rows <= 0 || b->q_lens[s] <= a.max_rows)) tiles += ceil_div64((int64_t)b->q_lens[s] * H, a.per_tile);
        a.tiles = (int)tiles;
        const int rc = split(tiles, 128);
        if (rc) return rc;
        launch_latent<RT>(be, a, mt, dim3(a.tiles, a.pieces));
        VX_CHECK_LAUNCH();
        merge();
        VX_CHECK_LAUNCH();
    }
    if (one > 0) {
        const int mt = query_tiles(H), across = ceil_div(H, mt * 16);
        a.decode = 1;
        const int rc = split(one * across, 64);
        if (rc) return rc;
        launch_latent<RT>(be, a, mt, dim3(a.pieces, b->n_seqs, across));
        VX_CHECK_LAUNCH();
        merge();
        VX_CHECK_LAUNCH();
    }
    return VX_OK;
}

// ---------------------------------------------------------------- angles, what a token leaves
__global__ void __launch_bounds__(256) rotary_table_kernel(const int32_t *pos, int rows, int pairs, const double *freqs, float factor, float *out) {
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (id >= (int64_t)rows * pairs) return;
    const double turn = 6.283185307179586476925286766559, a = pos[id / pairs] * freqs[id % pairs];
    float s, c;
    sincosf((float)(a - turn * rint(a / turn)), &s, &c);
    out[2 * id] = c * factor;
    out[2 * id + 1] = s * factor;
}

struct StoreArgs {
    vx_latent_store_args p;
    const int32_t *slot_mapping;
    int row_elems, pad;
};

template <typename T>
__global__ void __launch_bounds__(256) latent_store_kernel(StoreArgs a) {
    __shared__ float sm[4];
    const vx_latent_store_args &p = a.p;
    const int r = blockIdx.x, tid = threadIdx.x;
    const float *y = p.y + (size_t)r * p.ldy;
    const auto at = [&](int c) {
        float v = y[c];
        for (int s = 1; s < p.y_slices; s++) v += y[(size_t)s * p.y_stride + c];
        return v;
    };
    const auto normed = [&](int col, int n, const float *w, T *out) {
        constexpr int NV = 8;  // up to 2048 columns stay in registers
        float v[NV], ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = tid + i * 256;
            v[i] = c < n ? at(col + c) : 0.f;
            ss = fmaf(v[i], v[i], ss);
        }
        for (int c = tid + NV * 256; c < n; c += 256) {
            const float t = at(col + c);
            ss = fmaf(t, t, ss);
        }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        __syncthreads();  // (an earlier use of sm is over)
        if ((tid & 63) == 0) sm[tid >> 6] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf((sm[0] + sm[1] + sm[2] + sm[3]) / (float)n + p.eps);
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = tid + i * 256;
            if (c < n) out[c] = (T)(v[i] * inv * w[c]);
        }
        for (int c = tid + NV * 256; c < n; c += 256) out[c] = (T)(at(col + c) * inv * w[c]);
    };
    if (p.rank > 0) {
        T *dst = (T *)p.pool + (size_t)a.slot_mapping[r] * a.row_elems;
        for (int i = tid; i < p.rot_dim / 2; i += 256) {
            const float *cs = p.rot_tab + ((size_t)r * (p.rot_dim / 2) + i) * 2;
            const float u = at(p.kr_col + 2 * i), w = at(p.kr_col + 2 * i + 1);
            dst[a.pad + 2 * i] = (T)(u * cs[0] - w * cs[1]);
            dst[a.pad + 2 * i + 1] = (T)(w * cs[0] + u * cs[1]);
        }
        normed(p.c_col, p.rank, p.w_c, dst);
    }
    if (p.q_rank > 0) {
        T *dst = (T *)p.q_out + (size_t)r * p.ldq;
        normed(p.q_col, p.q_rank, p.w_q, dst);
        for (int c = p.q_rank + tid; c < p.ldq; c += 256) dst[c] = (T)0.f;
    }
}

template <typename T>
__global__ void __launch_bounds__(256) latent_spread_kernel(const T *latents, int row_elems, int pad, int rot_dim, const int32_t *a_rows, int64_t n,
                                                            T *pool, int kv_heads, int kp, size_t block, int block_size, int first) {
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (id >= n) return;
    const int per = rot_dim / 2;
    const int i = (int)(id % per) * 2, g = (int)(id / per % kv_heads), r = (int)(id / ((int64_t)per * kv_heads));
    const T *src = latents + (size_t)a_rows[r] * row_elems + pad + i;
    T *dst = pool + (size_t)(r / block_size) * block + ((size_t)g * block_size + r % block_size) * kp + first + i;
    dst[0] = src[0], dst[1] = src[1];
}

}  // namespace

extern "C" {

int vx_latent_pad(int rank) {
    if (rank < 1) return -1;
    for (int pad = 64; pad <= 512; pad *= 2)
        if (rank <= pad) return pad;
    return (rank + 63) / 64 * 64;
}

int vx_latent_row(int rank, int rot_dim) {
    if (rank < 1 || rot_dim < 0) return -1;
    return vx_latent_pad(rank) + (rot_dim > 64 ? (rot_dim + 63) / 64 * 64 : 64);
}

int vx_rotary_table(vx_backend *be, const int32_t *token_pos, int rows, int pairs, const double *freqs, float factor, float *out) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(token_pos && rows >= 1 && pairs >= 1 && freqs && out, "vx_rotary_table: bad arguments");
    rotary_table_kernel<<<(unsigned)ceil_div64((int64_t)rows * pairs, 256), 256, 0, be->stream>>>(token_pos, rows, pairs, freqs, factor, out);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_latent_store(vx_backend *be, int act, const vx_ragged *b, const vx_latent_store_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_latent_store");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_latent_store: unknown activation type %d", act);
    VX_REQUIRE(p && p->y && p->y_slices >= 1 && p->rank >= 0 && p->q_rank >= 0 && p->rank + p->q_rank > 0, "vx_latent_store: bad arguments");
    VX_REQUIRE(p->rank == 0 || (p->w_c && p->pool && p->rot_dim >= 0 && p->rot_dim % 2 == 0 && (p->rot_dim == 0 || p->rot_tab) &&
                                p->c_col >= 0 && p->kr_col >= 0 && p->c_col + p->rank <= p->ldy && p->kr_col + p->rot_dim <= p->ldy),
               "vx_latent_store: bad latent");
    VX_REQUIRE(p->q_rank == 0 || (p->w_q && p->q_out && p->ldq >= p->q_rank && p->q_col >= 0 && p->q_col + p->q_rank <= p->ldy),
               "vx_latent_store: bad query latent");
    StoreArgs a{*p, b->slot_mapping, 0, 0};
    if (p->rank > 0) a.row_elems = vx_latent_row(p->rank, p->rot_dim), a.pad = vx_latent_pad(p->rank);
    if (act == VX_ACT_BF16)
        latent_store_kernel<bf16><<<b->rows, 256, 0, be->stream>>>(a);
    else
        latent_store_kernel<float><<<b->rows, 256, 0, be->stream>>>(a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_attn_latent_fast(int act, int block_size, int rank, int rot_dim) {
    return act == VX_ACT_BF16 && block_size == BS && rank >= 1 && rank <= 512 && rot_dim >= 0 && rot_dim <= 64;
}

int vx_attn_latent(vx_backend *be, int act, const vx_ragged *b, const vx_latent_attn_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_attn_latent");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_attn_latent: unknown activation type %d", act);
    VX_REQUIRE(p && p->heads >= 1 && p->heads <= 65535 && p->rank >= 1 && p->rot_dim >= 0 && p->q && (p->rot_dim == 0 || p->qr) && p->pool && p->out,
               "vx_attn_latent: bad arguments");
    VX_REQUIRE(p->rank <= 2048 && p->rot_dim <= 1024, "vx_attn_latent: latents of %d + %d (at most 2048 + 1024)", p->rank, p->rot_dim);
    const int pad = vx_latent_pad(p->rank), row = vx_latent_row(p->rank, p->rot_dim);
    VX_REQUIRE(p->ldq >= (int64_t)p->heads * pad && p->ldo >= (int64_t)p->heads * pad && p->qr_stride >= p->rot_dim &&
                   (p->rot_dim == 0 || p->ldqr >= (int64_t)(p->heads - 1) * p->qr_stride + p->rot_dim),
               "vx_attn_latent: bad strides");
    VX_REQUIRE(b->n_seqs <= 65535, "vx_attn_latent: %d sequences", b->n_seqs);
    VX_REQUIRE(b->rows <= 65535, "vx_attn_latent: %d rows in one step (at most 65535)", b->rows);
    if (vx_attn_latent_fast(act, b->block_size, p->rank, p->rot_dim)) {
        VX_REQUIRE(p->ldq % 8 == 0 && p->ldo % 4 == 0 && (uintptr_t)p->q % 16 == 0 && (uintptr_t)p->out % 16 == 0 && (uintptr_t)p->pool % 16 == 0 &&
                       (p->rot_dim == 0 || (p->ldqr % 8 == 0 && p->qr_stride % 16 == 0 && (uintptr_t)p->qr % 16 == 0)),
                   "vx_attn_latent: alignment");
        Args a;
        memset(&a, 0, sizeof a);
        a.p = *p;
        a.cu = b->cu_seqlens, a.pos = b->token_pos, a.rows = b->table_rows, a.kv_lens = b->kv_lens, a.tables = b->block_tables;
        a.n_seqs = b->n_seqs, a.max_blocks = b->max_blocks, a.one_token = b->q_lens ? 0 : 1;
        if (pad == 64) return run_latent<1>(be, a, b);
        if (pad == 128) return run_latent<2>(be, a, b);
        if (pad == 256) return run_latent<4>(be, a, b);
        return run_latent<8>(be, a, b);
    }
    PlainAttn t;
    memset(&t, 0, sizeof t);
    t.heads = t.group = p->heads;
    t.q[0] = {p->q, p->ldq, p->rank, 0, pad, pad};
    t.q[1] = {p->qr, p->ldqr, p->rot_dim, pad, row - pad, p->qr_stride};
    t.row = row, t.v_dim = p->rank;
    t.pool = p->pool, t.block = (int64_t)b->block_size * row, t.k_tok = row, t.v_tok = row, t.v_elem = 1;
    t.scale = p->scale, t.sink = p->sink, t.bias_len = 1;
    t.out_scale = 1.0f, t.out = p->out, t.ldo = p->ldo, t.out_head = pad, t.out_cols = pad;
    t.max_rows = p->max_rows;
    launch_plain(be, act, b, t);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_latent_spread(vx_backend *be, int act, const void *latent_pool, int rank, int rot_dim, const int32_t *a_rows, int rows, void *pool,
                     int kv_heads, int k_dim, int v_dim, int block_size, int first) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_latent_spread: unknown activation type %d", act);
    VX_REQUIRE(latent_pool && a_rows && pool && rows >= 1 && rank >= 1 && rot_dim >= 0 && rot_dim % 2 == 0 && kv_heads >= 1 && block_size >= 1 &&
                   first >= 0 && first + rot_dim <= k_dim && v_dim >= 1,
               "vx_latent_spread: bad arguments");
    if (rot_dim == 0) return VX_OK;
    const int64_t n = (int64_t)rows * kv_heads * (rot_dim / 2);
    const size_t block = vx_kv_block_elems(block_size, kv_heads, k_dim, v_dim);
    const int row = vx_latent_row(rank, rot_dim), pad = vx_latent_pad(rank), kp = (k_dim + 7) & ~7;
    if (act == VX_ACT_BF16)
        latent_spread_kernel<bf16><<<(unsigned)ceil_div64(n, 256), 256, 0, be->stream>>>((const bf16 *)latent_pool, row, pad, rot_dim, a_rows, n, (bf16 *)pool,
                                                                                        kv_heads, kp, block, block_size, first);
    else
        latent_spread_kernel<float><<<(unsigned)ceil_div64(n, 256), 256, 0, be->stream>>>((const float *)latent_pool, row, pad, rot_dim, a_rows, n,
                                                                                         (float *)pool, kv_heads, kp, block, block_size, first);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
