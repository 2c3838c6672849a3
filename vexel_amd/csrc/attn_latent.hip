// Latent attention for mixed batches: what a token leaves in the paged pool (vx_latent_store), causal attention over it
// (vx_attn_latent), and the spreading of the rotated key part for layers that spell their keys out (vx_latent_spread).
//
// A pool row is one token: c [pad] | rotated key part [64 or more]. All heads read the same rows, so a workgroup takes
// 16, 32 or 64 (row, head) pairs of one sequence through a piece of its keys, a tile of 64 or 128 keys at a time:
//   tile -> LDS (each wave brings a share of it, requested a tile ahead into registers)
//   S^T = K Q^T       waves split the tile's keys and the queries; the queries' operands stay in registers
//   running maximum   exchanged through LDS, the weights go to LDS as two bfloat16 parts (16 bits of the 24)
//   O^T += V^T P^T    V is the first part of the same rows, read transposed (ds_read_tr); waves split the dimensions
// Pieces leave partial results that a second launch merges, which also counts the sink.
#include <string.h>

#include <algorithm>

#include "attn_plain.h"

using namespace vx;

namespace {

constexpr int BS = 16;  // tokens of a block (matrix-core kernel)
constexpr int MAX_PIECES = 256;

struct Args {
    vx_latent_attn_args p;
    const int32_t *cu, *pos, *rows, *kv_lens, *tables;
    int n_seqs, max_blocks, one_token;
    int decode;               // items are the sequences that bring one row; otherwise tiles of the others
    int min_rows, max_rows, tiles;
    int pieces, goal, cap, n_rows;  // pieces: room for so many of a sequence; goal, cap: see piece_of
    float *partial;           // [row, or sequence][piece][head][pad], then the same of (maximum, sum)
};

// Keys of one piece of a sequence of `len` tokens: `goal` pieces of whole tiles, more where they would be longer than cap.
__device__ __forceinline__ int piece_of(const Args &a, int len) {
    const int n = (len + a.goal - 1) / a.goal;
    return (min(n, a.cap) + 127) & ~127;
}

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

// MT query tiles of 16, tiles of KT keys, DEPTH of them on the way at a time.
// NT: nobody else reads the keys (non-temporal loads).
template <int RT, int MT, int KT, int DEPTH, bool NT>
__global__ void __launch_bounds__(512, 2) latent_kernel(Args a) {
    constexpr int NW = 8, CPR = RT * 8 + 8;           // waves; 16-byte pieces of a pool row
    constexpr int WK = NW / MT, NK = KT / 16 / WK;    // waves over keys; 16-key tiles of a wave
    constexpr int KR = KT / NW;                       // rows that a wave brings
    constexpr int RPL = 8 / RT, LC = KR / RPL, LR = KR / 8;  // rows whose c one load takes; loads of c, of rotated parts
    constexpr int KK = RT * 2 + 2;                    // steps of 32 dimensions
    constexpr int TD = RT * 4 < NW ? 1 : RT * 4 / NW; // 16-dimension tiles of a wave
    constexpr int PS = KT + 8;                        // a query's weights in LDS
    static_assert(NK * WK * 16 == KT && KR % 8 == 0 && BS % KR == 0, "tile shape");
    // piece c of row r lies at r * CPR + (c ^ (r & 7)): rows are whole multiples of 128 bytes, so that a constant part of r & 7 or of
    // c & 7 is an exclusive or on the address
    __shared__ u32x4 s_k[KT * CPR];
    __shared__ bf16 s_hi[MT * 16 * PS], s_lo[MT * 16 * PS];
    __shared__ float s_max[WK][MT * 16], s_l[WK][MT * 16];
    const vx_latent_attn_args &p = a.p;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, kw = wave % WK, mw = wave / WK, li = lane & 15, lq = lane >> 4;
    const int H = p.heads;
    int seq, m_first, piece, row0, n;
    if (a.decode) {
        seq = blockIdx.x, piece = blockIdx.y, m_first = blockIdx.z * MT * 16, n = 1;  // (a sequence's pieces mostly share a die)
        row0 = a.one_token ? seq : a.cu[seq];
        if (!a.one_token && a.cu[seq + 1] - row0 != 1) return;
    } else {
        int ti, count;
        if (!item_of_seq(a.cu, a.n_seqs, MT * 16, a.min_rows, a.tiles - 1 - blockIdx.x, &seq, &ti, &count, H, a.max_rows)) return;
        piece = blockIdx.y, m_first = ti * MT * 16;
        row0 = a.cu[seq], n = a.cu[seq + 1] - row0;
    }
    const int pos0 = a.kv_lens[seq] - n, pairs = n * H;
    const int pos_hi = pos0 + min((m_first + MT * 16 - 1) / H, n - 1);
    const int per = a.pieces == 1 ? pos0 + n : piece_of(a, pos0 + n), k_lo = piece * per, k_hi = min(pos_hi + 1, k_lo + per);
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
    f32x4 o[MT][TD];
#pragma unroll
    for (int t = 0; t < MT; t++) {
        m[t] = -INFINITY;
#pragma unroll
        for (int v = 0; v < TD; v++) o[t][v] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    u32x4 pf[DEPTH][LC + LR];
    const u32x4 *pool = (const u32x4 *)p.pool;
    const int cr = lane / (RT * 8), cc = lane % (RT * 8), rr = lane >> 3, rc = RT * 8 + (lane & 7);  // row and piece of a lane
    auto fetch = [&](int k0, u32x4 *f) {              // a wave's rows lie inside one block
        const int r0 = k0 + wave * KR, blk = bt[min(r0 / BS, last_blk)];
        const u32x4 *src = pool + ((size_t)blk * BS + r0 % BS) * CPR;
#pragma unroll
        for (int i = 0; i < LC; i++) {
            const u32x4 *e = src + (i * RPL + cr) * CPR + cc;
            f[i] = NT ? __builtin_nontemporal_load(e) : *e;
        }
#pragma unroll
        for (int i = 0; i < LR; i++) {
            const u32x4 *e = src + (i * 8 + rr) * CPR + rc;
            f[LC + i] = NT ? __builtin_nontemporal_load(e) : *e;
        }
    };
    char *const lds = (char *)s_k;
    const int put_c = ((wave * KR + cr) * CPR + (cc ^ (cr & 7))) * 16, put_r = ((wave * KR + rr) * CPR + (rc ^ rr)) * 16;
    const int get_k = (((kw * NK) * 16 + li) * CPR + (lq ^ (li & 7))) * 16;
    // transposed reads: rows 8 lq + 4 half + (li >> 2) of 32, pieces 2 (wave * TD + v) + ((li & 3) >> 1)
    const int get_v = ((lq * 8 + (li >> 2)) * CPR + (((li & 3) >> 1) ^ (li >> 2))) * 16 + (li & 1) * 8;
#pragma unroll
    for (int h = 0; h < DEPTH; h++)
        if (k_lo + h * KT < k_hi) fetch(k_lo + h * KT, pf[h]);
    auto tile = [&](int k0, u32x4 *f) {
#pragma unroll
        for (int i = 0; i < LC; i++) *(u32x4 *)(lds + ((put_c ^ ((i * RPL & 7) * 16)) + i * RPL * CPR * 16)) = f[i];
#pragma unroll
        for (int i = 0; i < LR; i++) *(u32x4 *)(lds + put_r + i * 8 * CPR * 16) = f[LC + i];
        __syncthreads();
        if (k0 + DEPTH * KT < k_hi) fetch(k0 + DEPTH * KT, f);
        f32x4 s[NK];
        float mx = -INFINITY;
#pragma unroll
        for (int nk = 0; nk < NK; nk++) {
            f32x4 s0 = f32x4{0.f, 0.f, 0.f, 0.f}, s1 = s0;  // (two chains)
#pragma unroll
            for (int kk = 0; kk < KK; kk++) {
                const bf16x8 key = *(const bf16x8 *)(lds + (get_k ^ ((kk & 1) * 64)) + nk * 16 * CPR * 16 + (kk >> 1) * 128);
                if (kk & 1)
                    s1 = mma(key, qf[kk], s1);
                else
                    s0 = mma(key, qf[kk], s0);
            }
            s[nk] = s0 + s1;
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
        if (wave * TD < RT * 4) {
            if (__any(moved)) {
#pragma unroll
                for (int t = 0; t < MT; t++)
#pragma unroll
                    for (int v = 0; v < TD; v++) o[t][v] *= al[t];
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
                for (int v = 0; v < TD; v++) {
                    s16x8 vt;
#pragma unroll
                    for (int half = 0; half < 2; half++) {
                        const int c = (wave * TD + v) * 2;
                        const s16x4 x = read_transposed(lds + (get_v ^ ((c & 7) * 16) ^ (half * 64)) + (c >> 3) * 128 + (ks * 32 + half * 4) * CPR * 16);
#pragma unroll
                        for (int j = 0; j < 4; j++) vt[half * 4 + j] = x[j];
                    }
                    const bf16x8 vb = __builtin_bit_cast(bf16x8, vt);
#pragma unroll
                    for (int t = 0; t < MT; t++) o[t][v] = mma(vb, hi[t], o[t][v]);
#pragma unroll
                    for (int t = 0; t < MT; t++) o[t][v] = mma(vb, lo[t], o[t][v]);
                }
            }
        }
        __syncthreads();  // (the tile and the weights are done with)
    };
    for (int k0 = k_lo; k0 < k_hi; k0 += DEPTH * KT)
#pragma unroll
        for (int h = 0; h < DEPTH; h++)
            if (k0 + h * KT < k_hi) tile(k0 + h * KT, pf[h]);
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (lane < 16) s_l[kw][mw * 16 + lane] = l;
    __syncthreads();
    if (wave * TD >= RT * 4) return;
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
            for (int v = 0; v < TD; v++) store4(out + (wave * TD + v) * 16, o[t][v] * inv);
        } else {
            const size_t at = ((size_t)(a.decode ? seq : row0 + tok) * a.pieces + piece) * H + head;
            float *dst = a.partial + at * (RT * 64) + lq * 4;
#pragma unroll
            for (int v = 0; v < TD; v++) *(f32x4 *)(dst + (wave * TD + v) * 16) = o[t][v];
            if (wave == 0 && lq == 0) {
                float *ml = a.partial + (size_t)a.n_rows * H * a.pieces * (RT * 64) + at * 2;
                ml[0] = m[t], ml[1] = sum;
            }
        }
    }
}

// One (row, head): its pieces become one.
__global__ void __launch_bounds__(128) latent_merge_kernel(Args a, int pad) {
    __shared__ float s_w[MAX_PIECES];
    const int h = blockIdx.x, own = blockIdx.y, lane = threadIdx.x & 63;  // own: the partial results' row
    const int row = a.decode && !a.one_token ? a.cu[own] : own, seq = a.decode ? own : seq_of_row(a.cu, a.n_seqs, row);
    const int brings = a.one_token ? 1 : a.cu[seq + 1] - a.cu[seq];
    if (a.decode ? brings != 1 : (brings < a.min_rows || (a.max_rows > 0 && brings > a.max_rows))) return;
    const int n = a.pos[row] / piece_of(a, a.kv_lens[seq]) + 1, H = a.p.heads;
    const size_t at = (size_t)own * a.pieces * H + h;
    const float *src = a.partial + at * pad, *ml = a.partial + (size_t)a.n_rows * H * a.pieces * pad + at * 2;
    float m = -INFINITY, l = 0.f;
    for (int i = lane; i < n; i += 64) m = fmaxf(m, ml[(size_t)2 * i * H]);
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) m = fmaxf(m, __shfl_xor(m, off, 64));
    for (int i = lane; i < n; i += 64) {
        const float w = __builtin_amdgcn_exp2f(ml[(size_t)2 * i * H] - m);
        l = fmaf(ml[(size_t)2 * i * H + 1], w, l);
        if (threadIdx.x < 64) s_w[i] = w;
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) l += __shfl_xor(l, off, 64);
    __syncthreads();
    const float inv = 1.0f / (l + sink_term(a.p, h, m));
    for (int d = threadIdx.x * 4; d < pad; d += blockDim.x * 4) {
        f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
        for (int i = 0; i < n; i++) o += *(const f32x4 *)(src + (size_t)i * H * pad + d) * s_w[i];
        store4((bf16 *)a.p.out + (size_t)row * a.p.ldo + (size_t)h * pad + d, o * inv);
    }
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
    // Pieces, so that the launch fills the chip. The lengths may be known as a bound only (max_kv_len), so that a sequence's own
    // length decides about its pieces on the device.
    const auto split = [&](int64_t wgs, int cap) -> int {
        a.n_rows = a.decode ? b->n_seqs : b->rows;  // (single tokens: one row a sequence)
        const int64_t room = most / ((int64_t)a.n_rows * H * (pad + 2) * 4), tiles = ceil_div(b->max_kv_len, 128);
        const auto bounded = [&](int64_t n) { return (int)std::max<int64_t>(1, std::min({n, tiles, room, (int64_t)MAX_PIECES})); };
        a.goal = bounded(ceil_div64(256, wgs));
        a.pieces = bounded(std::max<int64_t>(a.goal, ceil_div(b->max_kv_len, cap)));
        a.cap = std::max(cap, ceil_div(ceil_div(b->max_kv_len, a.pieces), 128) * 128);
        if (a.pieces == 1) return VX_OK;
        const size_t bytes = (size_t)a.n_rows * H * a.pieces * (pad + 2) * 4;
        const int rc = ensure_ws(be, &be->attn_ws, &be->attn_ws_bytes, bytes, "attention");
        a.partial = (float *)be->attn_ws;
        be->split.batch = 0;  // (whatever an earlier call left there is gone)
        return rc;
    };
    const auto merge = [&]() {
        if (a.pieces > 1)
            latent_merge_kernel<<<dim3(H, a.n_rows), pad / 4 < 64 ? 64 : 128, 0, be->stream>>>(a, pad);
    };
    if (longest > 0) {
        const int mt = query_tiles(longest * H);
        a.decode = 0;
        int64_t tiles = 0;
        for (int s = 0; s < b->n_seqs; s++)
            if (b->q_lens[s] > 1 && (a.max_rows <= 0 || b->q_lens[s] <= a.max_rows)) tiles += ceil_div64((int64_t)b->q_lens[s] * H, mt * 16);
        a.tiles = (int)tiles;
        const int rc = split(tiles, 1 << 28);
        if (rc) return rc;
        const dim3 grid(a.tiles, a.pieces);
        if (mt == 1)
            latent_kernel<RT, 1, 128, 1, false><<<grid, 512, 0, be->stream>>>(a);
        else if (mt == 2)
            latent_kernel<RT, 2, 64, 2, false><<<grid, 512, 0, be->stream>>>(a);
        else
            latent_kernel<RT, 4, 64, 1, false><<<grid, 512, 0, be->stream>>>(a);
        VX_CHECK_LAUNCH();
        merge();
        VX_CHECK_LAUNCH();
    }
    if (one > 0) {
        const int across = ceil_div(H, 16);  // (more heads to a workgroup leave more partial results, which cost more than keys from L2)
        a.decode = 1;
        const int rc = split(one * across, 1024);
        if (rc) return rc;
        const dim3 grid(b->n_seqs, a.pieces, across);
        if (across == 1)
            latent_kernel<RT, 1, 128, 1, true><<<grid, 512, 0, be->stream>>>(a);
        else
            latent_kernel<RT, 1, 128, 1, false><<<grid, 512, 0, be->stream>>>(a);
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

// blockIdx.y: the key's latent and rotated part, or the query's latent. VEC: columns of a thread at a time (4: everything aligned).
template <typename T, int VEC>
__global__ void __launch_bounds__(256) latent_store_kernel(StoreArgs a) {
    typedef float F __attribute__((ext_vector_type(VEC)));
    typedef T V __attribute__((ext_vector_type(VEC)));
    __shared__ float sm[4];
    const vx_latent_store_args &p = a.p;
    const int r = blockIdx.x, tid = threadIdx.x;
    const bool query = p.rank == 0 || blockIdx.y == 1;
    const float *y = p.y + (size_t)r * p.ldy;
    const auto at = [&](int c) {
        float v = y[c];
        for (int s = 1; s < p.y_slices; s++) v += y[(size_t)s * p.y_stride + c];
        return v;
    };
    T *const out = query ? (T *)p.q_out + (size_t)r * p.ldq : (T *)p.pool + (size_t)a.slot_mapping[r] * a.row_elems;
    const int col = query ? p.q_col : p.c_col, n = query ? p.q_rank : p.rank;
    const float *w = query ? p.w_q : p.w_c;
    if (!query)
        for (int i = tid; i < p.rot_dim / 2; i += 256) {
            const float *cs = p.rot_tab + ((size_t)r * (p.rot_dim / 2) + i) * 2;
            const float u = at(p.kr_col + 2 * i), v = at(p.kr_col + 2 * i + 1);
            out[a.pad + 2 * i] = (T)(u * cs[0] - v * cs[1]);
            out[a.pad + 2 * i + 1] = (T)(v * cs[0] + u * cs[1]);
        }
    constexpr int NV = 2;  // vectors of a thread that stay in registers: 512 * VEC columns
    F v[NV];
    float ss = 0.f;
    const auto load = [&](int c) {
        F t = *(const F *)(y + col + c);
#pragma unroll 4
        for (int s = 1; s < p.y_slices; s++) t += *(const F *)(y + (size_t)s * p.y_stride + col + c);
        return t;
    };
    const auto square = [&](F t) {
#pragma unroll
        for (int e = 0; e < VEC; e++) ss = fmaf(t[e], t[e], ss);
    };
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const int c = (tid + i * 256) * VEC;
        if (c < n) {
            v[i] = load(c);
            square(v[i]);
        }
    }
    for (int c = (tid + NV * 256) * VEC; c < n; c += 256 * VEC) square(load(c));
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    if ((tid & 63) == 0) sm[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((sm[0] + sm[1] + sm[2] + sm[3]) / (float)n + p.eps);
    const auto put = [&](int c, F t) {
        V o;
#pragma unroll
        for (int e = 0; e < VEC; e++) o[e] = (T)(t[e] * inv * w[c + e]);
        *(V *)(out + c) = o;
    };
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const int c = (tid + i * 256) * VEC;
        if (c < n) put(c, v[i]);
    }
    for (int c = (tid + NV * 256) * VEC; c < n; c += 256 * VEC) put(c, load(c));
    if (query)
        for (int c = n + tid; c < p.ldq; c += 256) out[c] = (T)0.f;
}

// A thread copies VEC neighbouring elements of one row to one head.
template <typename T, int VEC>
__global__ void __launch_bounds__(256) latent_spread_kernel(const T *latents, int row_elems, int pad, int rot_dim, const int32_t *a_rows, int64_t n,
                                                            T *pool, int kv_heads, int kp, size_t block, int block_size, int first) {
    typedef T V __attribute__((ext_vector_type(VEC)));
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (id >= n) return;
    const int per = rot_dim / VEC;
    const int i = (int)(id % per) * VEC, r = (int)(id / per % block_size + id / ((int64_t)per * block_size * kv_heads) * block_size);
    const int g = (int)(id / ((int64_t)per * block_size) % kv_heads);
    *(V *)(pool + (size_t)(r / block_size) * block + ((size_t)g * block_size + r % block_size) * kp + first + i) =
        *(const V *)(latents + (size_t)a_rows[r] * row_elems + pad + i);
}

template <typename T, int VEC>
void launch_spread(vx_backend *be, const void *latents, int row_elems, int pad, int rot_dim, const int32_t *a_rows, int rows, void *pool, int kv_heads,
                   int kp, size_t block, int block_size, int first) {
    const int64_t n = (int64_t)rows * kv_heads * (rot_dim / VEC);
    latent_spread_kernel<T, VEC><<<(unsigned)ceil_div64(n, 256), 256, 0, be->stream>>>((const T *)latents, row_elems, pad, rot_dim, a_rows, n, (T *)pool,
                                                                                      kv_heads, kp, block, block_size, first);
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
    const dim3 grid(b->rows, p->rank > 0 && p->q_rank > 0 ? 2 : 1);
    const bool wide = p->rank % 4 == 0 && p->q_rank % 4 == 0 && p->c_col % 4 == 0 && p->q_col % 4 == 0 && p->ldy % 4 == 0 && p->y_stride % 4 == 0 &&
                      p->ldq % 4 == 0 && (uintptr_t)p->y % 16 == 0 && (uintptr_t)p->pool % 16 == 0 && (uintptr_t)p->q_out % 16 == 0;
    if (act == VX_ACT_BF16 && wide)
        latent_store_kernel<bf16, 4><<<grid, 256, 0, be->stream>>>(a);
    else if (act == VX_ACT_BF16)
        latent_store_kernel<bf16, 1><<<grid, 256, 0, be->stream>>>(a);
    else
        latent_store_kernel<float, 1><<<grid, 256, 0, be->stream>>>(a);
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
                   first >= 0 && first % 2 == 0 && first + rot_dim <= k_dim && v_dim >= 1 && rows % block_size == 0,
               "vx_latent_spread: bad arguments");
    if (rot_dim == 0) return VX_OK;
    const size_t block = vx_kv_block_elems(block_size, kv_heads, k_dim, v_dim);
    const int row = vx_latent_row(rank, rot_dim), pad = vx_latent_pad(rank), kp = (k_dim + 7) & ~7;
    const bool wide = rot_dim % 8 == 0 && first % 8 == 0 && block % 8 == 0 && (uintptr_t)latent_pool % 16 == 0 && (uintptr_t)pool % 16 == 0;
    if (act == VX_ACT_F32)
        launch_spread<float, 2>(be, latent_pool, row, pad, rot_dim, a_rows, rows, pool, kv_heads, kp, block, block_size, first);
    else if (wide)
        launch_spread<bf16, 8>(be, latent_pool, row, pad, rot_dim, a_rows, rows, pool, kv_heads, kp, block, block_size, first);
    else
        launch_spread<bf16, 2>(be, latent_pool, row, pad, rot_dim, a_rows, rows, pool, kv_heads, kp, block, block_size, first);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
