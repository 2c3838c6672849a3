// Linear attention with a forget gate per channel over mixed batches (vx_forget_attn), and the norm of every head behind it
// (vx_head_norm). The gate f decides what stays and 1 - f what is written; the kernels are given g = 1 - f, so that a gate close to 1
// keeps its distance from it.
//
//  * step_kernel: sequences that bring few rows (and everything in float32 batches). A workgroup keeps 32 columns of one head's
//    state in registers and walks the rows; bound by reading and writing the state.
//  * Sequences with more rows, on the bfloat16 matrix cores, in chunks of four blocks of 16 rows:
//      prepare_kernel  per chunk and head: queries decayed from the chunk's start on, keys decayed to its end, the chunk's whole decay,
//                      and the scores of its rows among each other. All decays are running products of gates, never larger than 1:
//                      inside a block one by one, between blocks as what is left from the key to its block's end, of the blocks
//                      between, and from the query's block's start on.
//      walk_kernel     32 columns of one head's state in registers run over the chunks: outputs from the state and from the scores,
//                      then the state itself.
//    Float32 operands enter the products as two bfloat16 parts (16 bits of the 24).
#include <algorithm>

#include "state_tiles.h"

using namespace vx;

namespace {

constexpr int FEW = 16;        // rows of a sequence up to which it is walked
constexpr int CH = 64, SB = 16, NB = CH / SB;
constexpr int TS = 8;          // rows staged at a time by step_kernel
constexpr int VC = 32;         // state columns of a workgroup

struct ForgetArgs {
    vx_forget_args p;
    const int32_t *cu, *pos, *slots;
    int n_seqs, one_token;
    int max_rows;     // step_kernel: sequences with more rows are left out
    char *ws;         // per chunk and head: see Chunk
};

// What prepare_kernel leaves for a chunk of one head, in tiles of 16 x 32 in the order in which a wave's lanes hold an operand: element (r,
// c) of a tile at lane r + 16 (c / 8), place c % 8.
template <int DIM> struct Chunk {
    bf16 q_hi[NB][DIM / 32][512], q_lo[NB][DIM / 32][512];         // decayed queries: rows x channels
    bf16 k_hi[DIM / 16][CH / 32][512], k_lo[DIM / 16][CH / 32][512];  // decayed keys: channels x rows
    bf16 a_hi[NB][CH / 32][512], a_lo[NB][CH / 32][512];           // scores: rows x keys; tiles above the diagonal are not written
    float decay[DIM];
};
__device__ __forceinline__ int in_tile(int r, int c) { return ((r & 15) + ((c & 31) >> 3) * 16) * 8 + (c & 7); }

// ---------------------------------------------------------------- few rows
// Thread: columns 4 (tid % 8) .. of the workgroup's 32, state rows tid / 8 + 32 i.
template <typename T, int RD>
__global__ void __launch_bounds__(256) step_kernel(ForgetArgs a) {
    extern __shared__ float s_dyn[];  // q [TS][dim] | g [TS][dim] | v [TS][32] | partial outputs [TS][4][32]
    const vx_forget_args &p = a.p;
    const int seq = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * VC, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int row0 = a.one_token ? seq : a.cu[seq], len = a.one_token ? 1 : a.cu[seq + 1] - row0;
    if (len > a.max_rows) return;
    const int cols = min(VC, p.vdim - c0), c = tid & 7, d0 = tid >> 3;
    const bool live = c * 4 < cols;
    float *sq = s_dyn, *sg = sq + TS * p.dim, *sv = sg + TS * p.dim, *so = sv + TS * VC;
    float *state = p.state + (((size_t)a.slots[seq] * p.heads + h) * p.dim + d0) * p.vdim + c0 + c * 4;
    f32x4 S[RD];
    const bool old = a.pos[row0] > 0;
#pragma unroll
    for (int i = 0; i < RD; i++)
        S[i] = old && live && d0 + i * 32 < p.dim ? *(const f32x4 *)(state + (size_t)i * 32 * p.vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
    for (int t0 = 0; t0 < len; t0 += TS) {
        const int tn = min(TS, len - t0);
        __syncthreads();
        for (int i = tid; i < tn * p.dim; i += 256) {
            const int t = i / p.dim, d = i - t * p.dim;
            sq[i] = (float)((const T *)p.q)[(size_t)(row0 + t0 + t) * p.ldq + h * p.dim + d];
            sg[i] = p.g[(size_t)(row0 + t0 + t) * p.ldg + h * p.dim + d];
        }
        for (int i = tid; i < tn * VC; i += 256)
            sv[i] = (i & 31) < cols ? (float)((const T *)p.v)[(size_t)(row0 + t0 + (i >> 5)) * p.ldv + h * p.vdim + c0 + (i & 31)] : 0.f;
        __syncthreads();
        for (int t = 0; t < tn; t++) {
            const f32x4 v = *(const f32x4 *)(sv + t * VC + c * 4);
            f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < RD; i++) {
                const int d = min(d0 + i * 32, p.dim - 1);
                const float g = sg[t * p.dim + d], q = d0 + i * 32 < p.dim ? sq[t * p.dim + d] : 0.f;
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    S[i][e] = fmaf(g, v[e] - S[i][e], S[i][e]);
                    o[e] = fmaf(q, S[i][e], o[e]);
                }
            }
#pragma unroll
            for (int e = 0; e < 4; e++) {
                o[e] += __shfl_xor(o[e], 8, 64);
                o[e] += __shfl_xor(o[e], 16, 64);
                o[e] += __shfl_xor(o[e], 32, 64);
            }
            if (lane < 8) *(f32x4 *)(so + (t * 4 + wave) * VC + lane * 4) = o;
        }
        __syncthreads();
        for (int i = tid; i < tn * VC; i += 256) {
            const int t = i >> 5, x = i & 31;
            if (x < cols)
                p.out[(size_t)(row0 + t0 + t) * p.ldo + h * p.vdim + c0 + x] =
                    so[(t * 4) * VC + x] + so[(t * 4 + 1) * VC + x] + so[(t * 4 + 2) * VC + x] + so[(t * 4 + 3) * VC + x];
        }
    }
#pragma unroll
    for (int i = 0; i < RD; i++)
        if (live && d0 + i * 32 < p.dim) *(f32x4 *)(state + (size_t)i * 32 * p.vdim) = S[i];
}

// ---------------------------------------------------------------- many rows
// Sum over the 16 lanes that share lane / 16.
__device__ __forceinline__ float sum16(float v) {
#define VX_ROW_ROR(n) __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x120 + n, 0xf, 0xf, false))
    v += VX_ROW_ROR(8);
    v += VX_ROW_ROR(4);
    v += VX_ROW_ROR(2);
    v += VX_ROW_ROR(1);
#undef VX_ROW_ROR
    return v;
}

__device__ __forceinline__ bf16x8 scaled_hi(bf16x8 hi, bf16x8 lo, const float *m, bf16x8 *low) {
    bf16x8 h;
#pragma unroll
    for (int j = 0; j < 8; j++) {
        bf16 x, y;
        split(((float)hi[j] + (float)lo[j]) * m[j], &x, &y);
        h[j] = x, (*low)[j] = y;
    }
    return h;
}

// A thread works out the decays of one channel in one block, in registers; then the workgroup's waves share the scores. The scores inside
// blocks read the chunk's queries and gates from LDS, those between blocks the decayed queries and keys, in the same place.
template <int DIM>
__global__ void __launch_bounds__(NB * DIM) prepare_kernel(ForgetArgs a) {
    constexpr int LD = DIM + 8, LG = DIM + 4, DS = DIM / 16, WAVES = NB * DIM / 64;
    extern __shared__ float s_dyn[];
    float *s_e = s_dyn, *s_m = s_e + NB * DIM;           // decays of whole blocks [NB][DIM]; of the blocks between a pair: (2, 0), (3, 1), (3, 0)
    float *s_b = s_m + 3 * DIM;                          // of the blocks ahead of each [NB][DIM]
    float *s_g = s_b + NB * DIM;                         // 1 - gates [CH][LG]
    bf16 *s_q = (bf16 *)(s_g + CH * LG);                 // queries [CH][LD]
    bf16 *s_qh = (bf16 *)s_g, *s_ql = s_qh + CH * LD, *s_kh = s_ql + CH * LD, *s_kl = s_kh + CH * LD;
    const vx_forget_args &p = a.p;
    const int tid = threadIdx.x, lane = tid & 63, wave = wave_id(), h = blockIdx.y, l16 = lane & 15, q4 = (lane >> 4) * 4, q8 = (lane >> 4) * 8;
    int seq, ci, chunks;
    if (!item_of_seq(a.cu, a.n_seqs, CH, FEW + 1, blockIdx.x, &seq, &ci, &chunks)) return;
    const int row0 = a.cu[seq] + ci * CH, len = min(CH, a.cu[seq + 1] - row0);
    Chunk<DIM> &out = ((Chunk<DIM> *)a.ws)[(size_t)blockIdx.x * p.heads + h];
    const int d = tid % DIM, b = tid / DIM;
    bf16 q[SB];
    float g[SB];
#pragma unroll
    for (int j = 0; j < SB; j++) {  // (rows beyond the sequence: they keep everything and write nothing)
        const int t = b * SB + j, row = row0 + min(t, len - 1);
        q[j] = ((const bf16 *)p.q)[(size_t)row * p.ldq + h * DIM + d];
        g[j] = p.g[(size_t)row * p.ldg + h * DIM + d];
    }
    float keep = 1.f, left = 1.f, qd[SB], kd[SB];
#pragma unroll
    for (int j = 0; j < SB; j++) {
        const int t = b * SB + j;
        if (t >= len) q[j] = (bf16)0.f, g[j] = 0.f;
        s_q[t * LD + d] = q[j], s_g[t * LG + d] = g[j];
        keep *= 1.0f - g[j];
        qd[j] = (float)q[j] * keep;
    }
#pragma unroll
    for (int j = SB - 1; j >= 0; j--) {
        kd[j] = g[j] * left;
        left *= 1.0f - g[j];
    }
    s_e[b * DIM + d] = keep;
    __syncthreads();
    {
        float before = 1.f, after = 1.f;
#pragma unroll
        for (int k = 0; k < NB; k++) {
            const float e = s_e[k * DIM + d];
            if (k < b) before *= e;
            if (k > b) after *= e;
        }
        if (b == 0) {
            const float e1 = s_e[DIM + d], e2 = s_e[2 * DIM + d];
            s_m[d] = e1, s_m[DIM + d] = e2, s_m[2 * DIM + d] = e1 * e2;
            out.decay[d] = keep * after;
        }
        s_b[b * DIM + d] = before;
        bf16x8 kh[2], kl[2];
#pragma unroll
        for (int j = 0; j < SB; j++) {
            bf16 x, y;
            split(kd[j] * after, &x, &y);
            kh[j >> 3][j & 7] = x, kl[j >> 3][j & 7] = y;
        }
#pragma unroll
        for (int x = 0; x < 2; x++) {
            const int at = in_tile(d, b * SB + x * 8);
            *(bf16x8 *)&out.k_hi[d >> 4][b >> 1][at] = kh[x];
            *(bf16x8 *)&out.k_lo[d >> 4][b >> 1][at] = kl[x];
        }
    }
    // scores inside blocks: 16 lanes take one key, DS channels each, through the block's rows from the key's own on; a wave takes four
    // neighbouring keys
    for (int u = wave; u < NB * SB / 4; u += WAVES) {
        const int blk = u >> 2, s = (u & 3) * 4 + (lane >> 4), slice = l16 * DS, first = (u & 3) * 4;
        const float *gp = s_g + blk * SB * LG + slice;
        const bf16 *qp = s_q + blk * SB * LD + slice;
        float w[DS], own = 0.f;
#pragma unroll
        for (int e = 0; e < DS; e++) w[e] = gp[s * LG + e];
        for (int t = first; t < SB; t++) {
            float dot = 0.f;
#pragma unroll
            for (int e = 0; e < DS; e++) {
                const float gt = t > s ? gp[t * LG + e] : 0.f;
                w[e] = fmaf(-gt, w[e], w[e]);
                dot = fmaf((float)qp[t * LD + e], w[e], dot);
            }
            dot = sum16(dot);
            if (l16 == t && t >= s) own = dot;
        }
        bf16 x, y;
        split(own, &x, &y);
        const int at = in_tile(l16, blk * SB + s);
        out.a_hi[blk][blk >> 1][at] = x, out.a_lo[blk][blk >> 1][at] = y;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < SB; j++) {
        const int t = b * SB + j;
        bf16 x, y;
        split(qd[j], &x, &y);
        s_qh[t * LD + d] = x, s_ql[t * LD + d] = y;
        split(kd[j], &x, &y);
        s_kh[t * LD + d] = x, s_kl[t * LD + d] = y;
    }
    __syncthreads();
    // scores between blocks: a wave takes queries of block bi and keys of block bj
    for (int u = wave; u < 8; u += WAVES) {
        if (u >= 6) {  // above the diagonal, where a pair of blocks is read together
            const int bi = (u - 6) * 2;
            const bf16x4 zero = bf16x4{(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f};
            const int at = in_tile(l16, (bi + 1) * SB + q4);
            *(bf16x4 *)&out.a_hi[bi][bi >> 1][at] = zero;
            *(bf16x4 *)&out.a_lo[bi][bi >> 1][at] = zero;
            continue;
        }
        const int bi = u < 1 ? 1 : u < 3 ? 2 : 3, bj = u < 1 ? 0 : u < 3 ? u - 1 : u - 3;
        const float *m = bi - bj < 2 ? nullptr : s_m + (bi - bj == 3 ? 2 : bj) * DIM;
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < DIM; c += 32) {
            const int at_q = (bi * SB + l16) * LD + c + q8, at_k = (bj * SB + l16) * LD + c + q8;
            bf16x8 qh = *(const bf16x8 *)(s_qh + at_q), ql = *(const bf16x8 *)(s_ql + at_q);
            const bf16x8 kh = *(const bf16x8 *)(s_kh + at_k), kl = *(const bf16x8 *)(s_kl + at_k);
            if (m) {
                bf16x8 low;
                qh = scaled_hi(qh, ql, m + c + q8, &low);
                ql = low;
            }
            acc = mma(kl, qh, acc);
            acc = mma(kh, ql, acc);
            acc = mma(kh, qh, acc);
        }
        bf16x4 hi, lo;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            bf16 x, y;
            split(acc[r], &x, &y);
            hi[r] = x, lo[r] = y;
        }
        const int at = in_tile(l16, bj * SB + q4);
        *(bf16x4 *)&out.a_hi[bi][bj >> 1][at] = hi;
        *(bf16x4 *)&out.a_lo[bi][bj >> 1][at] = lo;
    }
    // the queries, decayed from the chunk's start on: a wave writes whole tiles
    for (int u = wave; u < NB * DIM / 32; u += WAVES) {
        const int blk = u / (DIM / 32), c = u % (DIM / 32) * 32 + q8, at = (blk * SB + l16) * LD + c;
        bf16x8 lo;
        const bf16x8 hi = scaled_hi(*(const bf16x8 *)(s_qh + at), *(const bf16x8 *)(s_ql + at), s_b + blk * DIM + c, &lo);
        *(bf16x8 *)&out.q_hi[blk][c >> 5][lane * 8] = hi;
        *(bf16x8 *)&out.q_lo[blk][c >> 5][lane * 8] = lo;
    }
}

// Waves 0 .. 3: the outputs of a block of rows each. Waves 4 .. 7: the state, every fourth tile of 16 channels. The state before a chunk
// and the chunk's values pass through LDS, in two buffers that take turns; what comes from memory is read AHEAD chunks ahead.
constexpr int AHEAD = 3;

template <int DT>
__global__ void __launch_bounds__(512) walk_kernel(ForgetArgs a) {
    constexpr int DIM = DT * 32, LD = DIM + 8, LV = VC + 8, TILES = DIM / 16, TP = (TILES + 3) / 4, NV = VC / 16;
    __shared__ bf16 s_h[2][VC * LD], s_l[2][VC * LD], s_v[2][CH * LV];
    const vx_forget_args &p = a.p;
    const int tid = threadIdx.x & 255, lane = tid & 63, wave = wave_id() & 3, h = blockIdx.y, v0 = blockIdx.z * VC;
    const int l16 = lane & 15, q4 = (lane >> 4) * 4, q8 = (lane >> 4) * 8, seq = blockIdx.x;
    const int row0 = a.cu[seq], rows = a.cu[seq + 1] - row0, chunks = (rows + CH - 1) / CH;
    if (rows <= FEW) return;
    int first = 0;
    for (int s = 0; s < seq; s++) {
        const int n = a.cu[s + 1] - a.cu[s];
        if (n > FEW) first += (n + CH - 1) / CH;
    }
    const Chunk<DIM> *chunk = (const Chunk<DIM> *)a.ws + (size_t)first * p.heads + h;
    const int cols = min(VC, p.vdim - v0);
    if (wave_id() < 4) {
        struct {
            bf16x8 qh[DT], ql[DT], ah[2], al[2];
        } op[AHEAD];
        const auto fetch = [&](int c, auto &o) {
            const Chunk<DIM> &k = chunk[(size_t)min(c, chunks - 1) * p.heads];
#pragma unroll
            for (int i = 0; i < DT; i++) {
                o.qh[i] = *(const bf16x8 *)&k.q_hi[wave][i][lane * 8];
                o.ql[i] = *(const bf16x8 *)&k.q_lo[wave][i][lane * 8];
            }
#pragma unroll
            for (int i = 0; i < 2; i++) {
                if (i * 2 > wave) break;
                o.ah[i] = *(const bf16x8 *)&k.a_hi[wave][i][lane * 8];
                o.al[i] = *(const bf16x8 *)&k.a_lo[wave][i][lane * 8];
            }
        };
        const auto step = [&](int c, auto &o) {
            const bf16 *sh = s_h[c & 1], *sl = s_l[c & 1], *sv = s_v[c & 1];
            __syncthreads();
            f32x4 acc[NV];
#pragma unroll
            for (int n = 0; n < NV; n++) {
                acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int k = 0; k < DT; k++) {
                    const int at = (n * 16 + l16) * LD + k * 32 + q8;
                    const bf16x8 hi = *(const bf16x8 *)(sh + at), lo = *(const bf16x8 *)(sl + at);
                    acc[n] = mma(lo, o.qh[k], acc[n]);
                    acc[n] = mma(hi, o.ql[k], acc[n]);
                    acc[n] = mma(hi, o.qh[k], acc[n]);
                }
#pragma unroll
                for (int k = 0; k < 2; k++) {
                    if (k * 2 > wave) break;
                    const bf16x8 vt = column8(sv, LV, k * 32, n * 16, lane);
                    acc[n] = mma(vt, o.al[k], acc[n]);
                    acc[n] = mma(vt, o.ah[k], acc[n]);
                }
            }
            if (c + AHEAD < chunks) fetch(c + AHEAD, o);
            const int t = c * CH + wave * 16 + l16;
            if (t >= rows) return;
            float *out = p.out + (size_t)(row0 + t) * p.ldo + h * p.vdim + v0 + q4;
#pragma unroll
            for (int n = 0; n < NV; n++)
                if (n * 16 < cols) *(f32x4 *)(out + n * 16) = acc[n];
        };
#pragma unroll
        for (int i = 0; i < AHEAD; i++) fetch(i, op[i]);
        for (int c = 0; c < chunks; c += AHEAD)
#pragma unroll
            for (int i = 0; i < AHEAD; i++)
                if (c + i < chunks) step(c + i, op[i]);
        return;
    }
    float *state = p.state + ((size_t)a.slots[seq] * p.heads + h) * DIM * p.vdim + v0;
    // channels 16 tile + 4 (lane / 16) .. of tile wave + 4 x, columns 16 n + lane % 16
    f32x4 S[TP][NV];
    const bool old = a.pos[row0] > 0;
#pragma unroll
    for (int x = 0; x < TP; x++)
#pragma unroll
        for (int n = 0; n < NV; n++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int d = (wave + 4 * x) * 16 + q4 + r, c = n * 16 + l16;
                S[x][n][r] = old && d < DIM && c < cols ? state[(size_t)d * p.vdim + c] : 0.f;
            }
    const bf16 *vp = (const bf16 *)p.v + (size_t)row0 * p.ldv + h * p.vdim + v0;
    struct {
        bf16x8 kh[TP][2], kl[TP][2], v;
        f32x4 f[TP];
    } op[AHEAD];
    const auto fetch = [&](int c, auto &o) {
        const Chunk<DIM> &k = chunk[(size_t)min(c, chunks - 1) * p.heads];
        const int t = c * CH + (tid >> 2), col = (tid & 3) * 8;
#pragma unroll
        for (int e = 0; e < 8; e++) o.v[e] = (bf16)0.f;
        if (t < rows && col < cols) o.v = *(const bf16x8 *)(vp + (size_t)t * p.ldv + col);
#pragma unroll
        for (int x = 0; x < TP; x++) {
            const int tile = min(wave + 4 * x, TILES - 1);
#pragma unroll
            for (int i = 0; i < 2; i++) {
                o.kh[x][i] = *(const bf16x8 *)&k.k_hi[tile][i][lane * 8];
                o.kl[x][i] = *(const bf16x8 *)&k.k_lo[tile][i][lane * 8];
            }
            o.f[x] = *(const f32x4 *)&k.decay[tile * 16 + q4];
        }
    };
    const auto step = [&](int c, auto &o) {
        bf16 *sh = s_h[c & 1], *sl = s_l[c & 1], *sv = s_v[c & 1];
#pragma unroll
        for (int x = 0; x < TP; x++) {
            if (wave + 4 * x >= TILES) break;
#pragma unroll
            for (int n = 0; n < NV; n++) {
                bf16x4 hi, lo;
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    bf16 y, z;
                    split(S[x][n][r], &y, &z);
                    hi[r] = y, lo[r] = z;
                }
                const int at = (n * 16 + l16) * LD + (wave + 4 * x) * 16 + q4;
                *(bf16x4 *)(sh + at) = hi;
                *(bf16x4 *)(sl + at) = lo;
            }
        }
        *(bf16x8 *)(sv + (tid >> 2) * LV + (tid & 3) * 8) = o.v;
        __syncthreads();  // (the buffers written now were last read two chunks ago, before the barrier of the chunk between)
        bf16x8 vt[2][NV];
#pragma unroll
        for (int k = 0; k < 2; k++)
#pragma unroll
            for (int n = 0; n < NV; n++) vt[k][n] = column8(sv, LV, k * 32, n * 16, lane);
#pragma unroll
        for (int x = 0; x < TP; x++)
#pragma unroll
            for (int n = 0; n < NV; n++) {
                S[x][n] *= o.f[x];
#pragma unroll
                for (int k = 0; k < 2; k++) {
                    S[x][n] = mma(o.kl[x][k], vt[k][n], S[x][n]);
                    S[x][n] = mma(o.kh[x][k], vt[k][n], S[x][n]);
                }
            }
        if (c + AHEAD < chunks) fetch(c + AHEAD, o);
    };
#pragma unroll
    for (int i = 0; i < AHEAD; i++) fetch(i, op[i]);
    for (int c = 0; c < chunks; c += AHEAD)
#pragma unroll
        for (int i = 0; i < AHEAD; i++)
            if (c + i < chunks) step(c + i, op[i]);
#pragma unroll
    for (int x = 0; x < TP; x++)
#pragma unroll
        for (int n = 0; n < NV; n++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int d = (wave + 4 * x) * 16 + q4 + r, c = n * 16 + l16;
                if (d < DIM && c < cols) state[(size_t)d * p.vdim + c] = S[x][n][r];
            }
}

template <typename T>
void launch_step(vx_backend *be, const ForgetArgs &a) {
    const dim3 grid(a.n_seqs, a.p.heads, ceil_div(a.p.vdim, VC));
    const size_t lds = (size_t)TS * (2 * a.p.dim + 5 * VC) * 4;
    const int rd = ceil_div(a.p.dim, 32);
    if (rd <= 1)
        step_kernel<T, 1><<<grid, 256, lds, be->stream>>>(a);
    else if (rd <= 2)
        step_kernel<T, 2><<<grid, 256, lds, be->stream>>>(a);
    else if (rd <= 4)
        step_kernel<T, 4><<<grid, 256, lds, be->stream>>>(a);
    else if (rd <= 8)
        step_kernel<T, 8><<<grid, 256, lds, be->stream>>>(a);
    else
        step_kernel<T, 16><<<grid, 256, lds, be->stream>>>(a);
}

template <int DT>
int launch_chunks(vx_backend *be, ForgetArgs a, int chunks) {
    constexpr int DIM = DT * 32;
    constexpr size_t inside = (size_t)CH * (DIM + 4) * 4 + (size_t)CH * (DIM + 8) * 2, between = (size_t)4 * CH * (DIM + 8) * 2;
    constexpr size_t lds = (size_t)(2 * NB + 3) * DIM * 4 + (inside > between ? inside : between);
    const int rc = ensure_ws(be, &be->scan_ws, &be->scan_ws_bytes, (size_t)chunks * a.p.heads * sizeof(Chunk<DIM>), "scan");
    if (rc) return rc;
    a.ws = (char *)be->scan_ws;
    static bool allowed = false;
    if (!allowed) {
        (void)hipFuncSetAttribute((const void *)prepare_kernel<DIM>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        allowed = true;
    }
    prepare_kernel<DIM><<<dim3(chunks, a.p.heads), NB * DIM, lds, be->stream>>>(a);
    VX_CHECK_LAUNCH();
    walk_kernel<DT><<<dim3(a.n_seqs, a.p.heads, ceil_div(a.p.vdim, VC)), 512, 0, be->stream>>>(a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

// ---------------------------------------------------------------- norm of every head
// LANES lanes take a head of a row, four neighbouring columns each, again and again where it is wider.
template <typename T, int LANES>
__global__ void __launch_bounds__(256) head_norm_kernel(const float *x, int ldx, const float *w, float eps, int rows, int heads, int vdim, int count, T *out,
                                                        int ldo) {
    const int64_t id = ((int64_t)blockIdx.x * 256 + threadIdx.x) / LANES;
    const int row = (int)(id / (heads + 1)), h = (int)(id - (int64_t)row * (heads + 1)), l = threadIdx.x % LANES;
    if (row >= rows) return;  // (whole waves or whole heads: the shuffles stay within LANES lanes)
    T *o = out + (size_t)row * ldo;
    if (h == heads) {  // the columns that pad the row
        for (int c = heads * vdim + l; c < ldo; c += LANES) o[c] = (T)0.f;
        return;
    }
    const float *xr = x + (size_t)row * ldx + h * vdim;
    float ss = 0.f;
    for (int c = l * 4; c < vdim; c += LANES * 4) {
        const f32x4 v = *(const f32x4 *)(xr + c);
#pragma unroll
        for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
    }
#pragma unroll
    for (int off = LANES / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    const float inv = 1.0f / sqrtf(ss / (float)count + eps);
    for (int c = l * 4; c < vdim; c += LANES * 4) store4(o + h * vdim + c, *(const f32x4 *)(xr + c) * inv * *(const f32x4 *)(w + c));
}

template <typename T>
void launch_head_norm(vx_backend *be, const float *x, int ldx, const float *w, float eps, int rows, int heads, int vdim, int count, T *out, int ldo) {
    const auto grid = [&](int lanes) { return (unsigned)ceil_div64((int64_t)rows * (heads + 1) * lanes, 256); };
    if (vdim <= 32)
        head_norm_kernel<T, 8><<<grid(8), 256, 0, be->stream>>>(x, ldx, w, eps, rows, heads, vdim, count, out, ldo);
    else if (vdim <= 64)
        head_norm_kernel<T, 16><<<grid(16), 256, 0, be->stream>>>(x, ldx, w, eps, rows, heads, vdim, count, out, ldo);
    else if (vdim <= 128)
        head_norm_kernel<T, 32><<<grid(32), 256, 0, be->stream>>>(x, ldx, w, eps, rows, heads, vdim, count, out, ldo);
    else
        head_norm_kernel<T, 64><<<grid(64), 256, 0, be->stream>>>(x, ldx, w, eps, rows, heads, vdim, count, out, ldo);
}

}  // namespace

extern "C" {

int vx_forget_attn_fast(int act, int dim, int vdim) {
    return act == VX_ACT_BF16 && dim >= 32 && dim % 32 == 0 && dim <= 128 && vdim >= 16 && vdim % 16 == 0 && vdim <= 512;
}

int vx_forget_attn(vx_backend *be, int act, const vx_ragged *b, const vx_forget_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_forget_attn");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_forget_attn: unknown activation type %d", act);
    VX_REQUIRE(p && p->heads >= 1 && p->heads <= 65535 && p->dim >= 32 && p->dim % 32 == 0 && p->dim <= 512 && p->vdim >= 16 && p->vdim % 16 == 0 &&
                   p->vdim <= 512,
               "vx_forget_attn: bad heads");
    VX_REQUIRE(p->q && p->v && p->g && p->state && p->out, "vx_forget_attn: null argument");
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    VX_REQUIRE(p->ldq >= p->heads * p->dim && p->ldg >= p->heads * p->dim && p->ldv >= p->heads * p->vdim && p->ldo >= p->heads * p->vdim &&
                   p->ldq % 8 == 0 && p->ldv % 8 == 0 && p->ldo % 4 == 0 && al(p->q) && al(p->v) && al(p->state) && al(p->out),
               "vx_forget_attn: bad strides or alignment");
    ForgetArgs a{*p, b->cu_seqlens, b->token_pos, b->table_rows, b->n_seqs, b->q_lens ? 0 : 1, FEW, nullptr};
    const bool walk_all = !vx_forget_attn_fast(act, p->dim, p->vdim);
    bool few = !b->q_lens || walk_all, many = false;
    if (b->q_lens && !walk_all)
        for (int s = 0; s < b->n_seqs; s++) (b->q_lens[s] <= FEW ? few : many) = true;
    if (walk_all) a.max_rows = 1 << 30;
    if (many) {
        const int chunks = count_items(b, CH, FEW + 1);
        rc = p->dim == 32 ? launch_chunks<1>(be, a, chunks) : p->dim == 64 ? launch_chunks<2>(be, a, chunks) : p->dim == 96 ? launch_chunks<3>(be, a, chunks)
                                                                                                             : launch_chunks<4>(be, a, chunks);
        if (rc) return rc;
    }
    if (few) {
        if (act == VX_ACT_BF16)
            launch_step<bf16>(be, a);
        else
            launch_step<float>(be, a);
        VX_CHECK_LAUNCH();
    }
    return VX_OK;
}

int vx_head_norm(vx_backend *be, int act, const float *x, int ldx, const float *w, float eps, int rows, int heads, int vdim, int count, void *out,
                 int ldo) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_head_norm: unknown activation type %d", act);
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    VX_REQUIRE(x && w && out && rows >= 1 && heads >= 1 && vdim >= 4 && vdim % 4 == 0 && count >= 1 && count <= vdim && ldx >= heads * vdim &&
                   ldo >= heads * vdim && ldx % 4 == 0 && ldo % 4 == 0 && al(x) && al(w) && al(out),
               "vx_head_norm: bad arguments");
    if (act == VX_ACT_BF16)
        launch_head_norm<bf16>(be, x, ldx, w, eps, rows, heads, vdim, count, (bf16 *)out, ldo);
    else
        launch_head_norm<float>(be, x, ldx, w, eps, rows, heads, vdim, count, (float *)out, ldo);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
