// Causal grouped-query attention over a paged pool for mixed batches, with a per-head distance bias, a query temperature, a
// softmax sink per head, an output gate, a sliding window or chunks, a cap on the scores and differential heads
// (vx_attn_ragged).
//
//  * prefill_kernel: sequences that bring several rows. A wave owns QT x 16 (row, head) pairs of one K/V head and walks
//    the keys in groups of 32 (two 16-token blocks); the four waves of a workgroup walk the same keys.
//  * decode_kernel + merge_kernel: sequences that bring one row. A workgroup takes a piece of one sequence's keys for all
//    query heads of one K/V head, its waves every fourth group; the pieces' partial results are merged by a second
//    launch, which also applies the gate.
//  * attn_plain_kernel (attn_plain.h): one workgroup per (row, head), any geometry, and everything in float32 batches.
//    Differential heads: both maps' float32 results, combined by diff_kernel.
//
// Differential heads (MAPS 2): query tiles come in pairs, one per map, that meet the same V; the pair is combined where
// a row's result is written.
//
// Matrix products of the first two: S^T = K Q^T and O^T = V^T P^T on the bfloat16 matrix cores. The keys of a group are
// dealt to the two 16-row tiles of S^T so that a lane ends with eight consecutive keys of one query, which is the
// operand layout of the second product; V lies transposed in the pool, so that its operand is eight consecutive keys
// of one dimension as well, and nothing passes through LDS. The weights P are float32 and enter the second product as
// two bfloat16 parts (16 bits of the 24). Scores, bias, softmax and sums are float32.
#include <string.h>

#include <algorithm>

#include "attn_tiles.h"

using namespace vx;

namespace {

typedef AttnArgs Args;

template <int KD, int VD, int QT, int MAPS, bool NT>
__device__ __forceinline__ void group(const Args &a, Keys<KD, VD, MAPS, NT> &ks, Queries<KD, VD, QT> &qs, int k0, int next_b0, int next_b1,
                                      bool more, int lane, bool whole, bool distant, const float *s_lut) {
    f32x4 st[QT][2];
#pragma unroll
    for (int t = 0; t < QT; t++)
#pragma unroll
        for (int h = 0; h < 2; h++) {
            st[t][h] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KD; kk++) st[t][h] = mma(ks.k[t % MAPS][h][kk], qs.q[t][kk], st[t][h]);
        }
    if (more) ks.load_k(next_b0, next_b1);
#pragma unroll
    for (int t = 0; t < QT; t++) qs.template step<MAPS, NT>(a, ks, st[t][0], st[t][1], t, k0, lane, whole, distant, s_lut);
}

// bias tables of the workgroup's heads, times log2(e)
__device__ __forceinline__ void load_lut(const Args &a, int g, float *s_lut) {
    if (a.lut_lds) {
        const float *src = a.p.bias + (size_t)g * a.group * a.p.bias_len;
        for (int i = threadIdx.x; i < a.group * a.p.bias_len; i += blockDim.x) s_lut[i] = src[i] * kLog2e;
        __syncthreads();
    }
}

// What the difference of two maps' results is multiplied with. diff(v): columns v * 16 + 4 (lane / 16) .. of it; the head's columns lie
// in the four lanes lane % 16 + 16 i.
template <int VD, class O>
__device__ __forceinline__ float diff_factor(const Args &a, int lane, O &&diff) {
    float ss = 0.f;
#pragma unroll
    for (int v = 0; v < VD; v++) {
        const f32x4 d = diff(v);
        const int c = v * 16 + (lane >> 4) * 4;
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (c + r < a.p.v_dim) ss = fmaf(d[r], d[r], ss);
    }
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    return a.p.diff_scale / sqrtf(ss / (float)a.p.v_dim + a.p.diff_eps);
}

// The four waves of a workgroup: 4 / KS groups of QT x 16 queries (of QT / MAPS x 16 (row, head) pairs), KS waves to a group that
// take turns at the key groups.
template <int KD, int VD, int QT, int KS, int MAPS>
__global__ void __launch_bounds__(256) prefill_kernel(Args a) {
    extern __shared__ float s_dyn[];
    constexpr int RG = 4 / KS, LDO = VD * 16 + 4, PT = QT / MAPS;
    __shared__ float s_m[RG][KS][QT * 16], s_l[RG][KS][QT * 16];
    float *s_lut = s_dyn;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, rg = wave / KS, ks_id = wave % KS;
    const int g = blockIdx.x % a.p.kv_heads, id = a.tiles - 1 - blockIdx.x / a.p.kv_heads;  // late tiles, the longest, first
    int seq, ti, count;
    if (!item_of_seq(a.cu, a.n_seqs, a.tile_rows, a.min_rows, id, &seq, &ti, &count)) return;
    load_lut(a, g, s_lut);
    const int row0 = a.cu[seq] + ti * a.tile_rows, ntok = min(a.tile_rows, a.cu[seq + 1] - row0);
    const int pos0 = a.pos[row0];
    const int m_first = rg * 16 * PT;
    const bool any = m_first < ntok * a.group;  // the group has queries (the last tile of a sequence may be short)
    if (KS == 1 && !any) return;                // (no barrier follows)
    const int32_t *bt = a.tables + (size_t)a.rows[seq] * a.max_blocks;
    const int t_lo = min(m_first / a.group, ntok - 1), t_hi = min((m_first + 16 * PT - 1) / a.group, ntok - 1);
    const int pos_lo = pos0 + t_lo, pos_hi = pos0 + t_hi, last_blk = pos_hi / BS, groups = any ? pos_hi / 32 + 1 : 0;
    const int g_first = first_key(a.p, pos_lo) / 32, all_from = first_key(a.p, pos_hi);

    Queries<KD, VD, QT> qs;
    qs.clear();
    int tok[QT], head[QT];
#pragma unroll
    for (int t = 0; t < QT; t++) {
        const int m = m_first + t / MAPS * 16 + (lane & 15), map = t % MAPS;
        tok[t] = m / a.group, head[t] = g * a.group + m % a.group;
        const int tt = min(tok[t], ntok - 1);
        qs.pos[t] = pos0 + tt;
        qs.lo[t] = first_key(a.p, pos0 + tt);
        qs.lut[t] = (a.lut_lds ? m % a.group : head[t]) * a.p.bias_len;
        qs.qs[t] = score_factor(a.p, qs.pos[t]);
        qs.far[t] = score_offset(a.p, head[t]);
        const bf16 *q = (const bf16 *)a.p.q + (size_t)(row0 + tt) * a.p.ldq + (head[t] * MAPS + map) * a.p.k_dim;
#pragma unroll
        for (int kk = 0; kk < KD; kk++) qs.q[t][kk] = load_q(q, kk * 32 + (lane >> 4) * 8, a.p.k_dim, a.vec_q);
    }
    Keys<KD, VD, MAPS, false> ks;
    ks.init(a, g, lane);
    int gi = g_first + ks_id;
    if (gi < groups) {
        int b0 = bt[min(2 * gi, last_blk)], b1 = bt[min(2 * gi + 1, last_blk)];
        ks.load_k(b0, b1);
        for (; gi < groups; gi += KS) {
            ks.load_v(b0, b1, lane);
            const bool more = gi + KS < groups;
            if (more) b0 = bt[min(2 * (gi + KS), last_blk)], b1 = bt[min(2 * (gi + KS) + 1, last_blk)];
            const int k0 = gi * 32;
            group<KD, VD, QT, MAPS, false>(a, ks, qs, k0, b0, b1, more, lane, k0 + 31 <= pos_lo && k0 >= all_from, pos_lo - (k0 + 31) >= a.p.bias_len - 1, s_lut);
        }
    }
    float l[QT];
#pragma unroll
    for (int t = 0; t < QT; t++) {
        l[t] = qs.l[t];
        l[t] += __shfl_xor(l[t], 16, 64);
        l[t] += __shfl_xor(l[t], 32, 64);
    }
    if constexpr (KS == 1) {
        if constexpr (MAPS == 2) {
#pragma unroll
            for (int t = 0; t < QT; t += 2) {
                const float i1 = 1.0f / (l[t] + sink_term(a.p, head[t] * 2, qs.m[t]));
                const float i2 = a.p.diff_lambda / (l[t + 1] + sink_term(a.p, head[t] * 2 + 1, qs.m[t + 1]));
#pragma unroll
                for (int v = 0; v < VD; v++) qs.o[t][v] = qs.o[t][v] * i1 - qs.o[t + 1][v] * i2;
                const float f = diff_factor<VD>(a, lane, [&](int v) { return qs.o[t][v]; });
                if (tok[t] >= ntok) continue;
#pragma unroll
                for (int v = 0; v < VD; v++) write4(a, row0 + tok[t], head[t], v * 16 + (lane >> 4) * 4, qs.o[t][v] * f);
            }
            return;
        }
#pragma unroll
        for (int t = 0; t < QT; t++) {
            if (tok[t] >= ntok) continue;
            const float inv = 1.0f / (l[t] + sink_term(a.p, head[t], qs.m[t]));  // (a row sees itself: l > 0)
#pragma unroll
            for (int v = 0; v < VD; v++) write4(a, row0 + tok[t], head[t], v * 16 + (lane >> 4) * 4, qs.o[t][v] * inv);
        }
    } else {
        // the results of a group's waves become one
#pragma unroll
        for (int t = 0; t < QT; t++)
            if (lane < 16) s_m[rg][ks_id][t * 16 + lane] = qs.m[t], s_l[rg][ks_id][t * 16 + lane] = l[t];
        __syncthreads();  // (the bias tables in s_dyn are done with as well)
        float *s_o = s_dyn + rg * QT * 16 * LDO;
        float mg[QT];
#pragma unroll
        for (int t = 0; t < QT; t++) {
            mg[t] = -INFINITY;
#pragma unroll
            for (int w = 0; w < KS; w++) mg[t] = fmaxf(mg[t], s_m[rg][w][t * 16 + (lane & 15)]);
        }
        for (int w = 0; w < KS; w++) {
            if (ks_id == w) {
#pragma unroll
                for (int t = 0; t < QT; t++) {
                    const float f = qs.m[t] > -INFINITY ? __builtin_amdgcn_exp2f(qs.m[t] - mg[t]) : 0.f;
#pragma unroll
                    for (int v = 0; v < VD; v++) {
                        f32x4 *dst = (f32x4 *)(s_o + (t * 16 + (lane & 15)) * LDO + v * 16 + (lane >> 4) * 4);
                        const f32x4 x = qs.o[t][v] * f;
                        *dst = w == 0 ? x : *dst + x;
                    }
                }
            }
            __syncthreads();
        }
        if (!any) return;
        const auto total = [&](int t) {
            float sum = 0.f;
#pragma unroll
            for (int w = 0; w < KS; w++) {
                const float mw = s_m[rg][w][t * 16 + (lane & 15)];
                if (mw > -INFINITY) sum += s_l[rg][w][t * 16 + (lane & 15)] * __builtin_amdgcn_exp2f(mw - mg[t]);
            }
            return sum;
        };
        if constexpr (MAPS == 2) {
#pragma unroll
            for (int t = 0; t < QT; t += 2) {
                const float i1 = 1.0f / (total(t) + sink_term(a.p, head[t] * 2, mg[t]));
                const float i2 = a.p.diff_lambda / (total(t + 1) + sink_term(a.p, head[t] * 2 + 1, mg[t + 1]));
                const auto diff = [&](int v) {
                    const float *o = s_o + (t * 16 + (lane & 15)) * LDO + v * 16 + (lane >> 4) * 4;
                    return *(const f32x4 *)o * i1 - *(const f32x4 *)(o + 16 * LDO) * i2;
                };
                const float f = diff_factor<VD>(a, lane, diff);
                if (tok[t] >= ntok) continue;
                for (int v = ks_id; v < VD; v += KS) write4(a, row0 + tok[t], head[t], v * 16 + (lane >> 4) * 4, diff(v) * f);
            }
            return;
        }
#pragma unroll
        for (int t = 0; t < QT; t++) {
            if (tok[t] >= ntok) continue;
            const float inv = 1.0f / (total(t) + sink_term(a.p, head[t], mg[t]));
            for (int v = ks_id; v < VD; v += KS)
                write4(a, row0 + tok[t], head[t], v * 16 + (lane >> 4) * 4,
                       *(const f32x4 *)(s_o + (t * 16 + (lane & 15)) * LDO + v * 16 + (lane >> 4) * 4) * inv);
        }
    }
}

template <int KD, int VD, int MAPS>
__global__ void __launch_bounds__(256, VD <= 8 && MAPS * KD <= 6 ? 2 : 1) decode_kernel(Args a) {
    constexpr int QT = MAPS;
    extern __shared__ float s_dyn[];
    __shared__ float s_m[4][QT * 16], s_l[4][QT * 16];
    float *s_lut = s_dyn;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int g = blockIdx.x % a.p.kv_heads, h0 = blockIdx.x / a.p.kv_heads * 16;  // 16 of the group's query heads
    int seq, piece;
    if (a.items) {
        if ((int)blockIdx.y >= a.items[0]) return;
        seq = a.items[4 + 4 * blockIdx.y], piece = a.items[5 + 4 * blockIdx.y];
    } else {
        piece = blockIdx.y, seq = blockIdx.z;
    }
    const int row = a.one_token ? seq : a.cu[seq];
    if (!a.one_token && a.cu[seq + 1] - row != 1) return;
    const int len = a.kv_lens[seq], pos = len - 1, first = first_key(a.p, pos);
    const int start = first / 32 * 32, p_lo = (a.from_start ? 0 : start) + piece * a.piece, k_lo = max(p_lo, start), k_hi = min(len, p_lo + a.piece);
    if (k_lo >= k_hi) return;
    load_lut(a, g, s_lut);
    const int last_blk = pos / BS;
    const int32_t *bt = a.tables + (size_t)a.rows[seq] * a.max_blocks;

    Queries<KD, VD, QT> qs;
    qs.clear();
    const float factor = score_factor(a.p, pos);
#pragma unroll
    for (int t = 0; t < QT; t++) {
        const int hh = min(h0 + (lane & 15), a.group - 1), h = g * a.group + hh;
        qs.pos[t] = pos;
        qs.lo[t] = first;
        qs.lut[t] = (a.lut_lds ? hh : h) * a.p.bias_len;
        qs.qs[t] = factor;
        qs.far[t] = score_offset(a.p, h);
        const bf16 *q = (const bf16 *)a.p.q + (size_t)row * a.p.ldq + (h * MAPS + t) * a.p.k_dim;
#pragma unroll
        for (int kk = 0; kk < KD; kk++) qs.q[t][kk] = load_q(q, kk * 32 + (lane >> 4) * 8, a.p.k_dim, a.vec_q);
    }
    Keys<KD, VD, MAPS, true> ks;
    ks.init(a, g, lane);
    const int g_hi = (k_hi + 31) / 32;
    int gi = k_lo / 32 + wave;
    if (gi < g_hi) {
        int b0 = bt[min(2 * gi, last_blk)], b1 = bt[min(2 * gi + 1, last_blk)];
        ks.load_k(b0, b1);
        for (; gi < g_hi; gi += 4) {
            ks.load_v(b0, b1, lane);
            const bool more = gi + 4 < g_hi;
            if (more) b0 = bt[min(2 * gi + 8, last_blk)], b1 = bt[min(2 * gi + 9, last_blk)];
            const int k0 = gi * 32;
            group<KD, VD, QT, MAPS, true>(a, ks, qs, k0, b0, b1, more, lane, k0 + 31 <= pos && k0 >= first, pos - (k0 + 31) >= a.p.bias_len - 1, s_lut);
        }
    }
    // the four waves' results become one
#pragma unroll
    for (int t = 0; t < QT; t++) {
        float l = qs.l[t];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        if (lane < 16) s_m[wave][t * 16 + lane] = qs.m[t], s_l[wave][t * 16 + lane] = l;
    }
    __syncthreads();  // (the bias tables in s_dyn are done with as well)
    float *s_o = s_dyn;  // [QT * 16][VD * 16 + 4]
    constexpr int LDO = VD * 16 + 4;
    for (int w = 0; w < 4; w++) {
        if (wave == w) {
#pragma unroll
            for (int t = 0; t < QT; t++) {
                const int c = t * 16 + (lane & 15);
                const float mg = fmaxf(fmaxf(s_m[0][c], s_m[1][c]), fmaxf(s_m[2][c], s_m[3][c]));
                const float f = qs.m[t] > -INFINITY ? __builtin_amdgcn_exp2f(qs.m[t] - mg) : 0.f;
#pragma unroll
                for (int v = 0; v < VD; v++) {
                    f32x4 *dst = (f32x4 *)(s_o + c * LDO + v * 16 + (lane >> 4) * 4);
                    const f32x4 x = qs.o[t][v] * f;
                    *dst = w == 0 ? x : *dst + x;
                }
            }
        }
        __syncthreads();
    }
    const int vd = a.p.v_dim;
    for (int i = wave; i < MAPS * min(16, a.group - h0); i += 4) {
        const int hh = i / MAPS, c = i % MAPS * 16 + hh;
        float *dst = a.partial + ((((size_t)seq * a.p.heads + g * a.group + h0 + hh) * MAPS + i % MAPS) * a.pieces + piece) * (vd + 2);
        float mg = -INFINITY, l = 0.f;
        for (int w = 0; w < 4; w++) mg = fmaxf(mg, s_m[w][c]);
        for (int w = 0; w < 4; w++) l += s_m[w][c] > -INFINITY ? s_l[w][c] * __builtin_amdgcn_exp2f(s_m[w][c] - mg) : 0.f;
        if (lane == 0) dst[0] = mg, dst[1] = l;
        for (int d = lane; d < vd; d += 64) dst[2 + d] = s_o[c * LDO + d];
    }
}

template <int MAPS>
__global__ void __launch_bounds__(64) merge_kernel(Args a) {
    const int h = blockIdx.x, seq = blockIdx.y, vd = a.p.v_dim;
    const int row = a.one_token ? seq : a.cu[seq];
    if (!a.one_token && a.cu[seq + 1] - row != 1) return;
    const int len = a.kv_lens[seq], start = first_key(a.p, len - 1) / 32 * 32, skip = a.from_start ? start / a.piece : 0;  // pieces nobody sees
    const int n = (len - (a.from_start ? skip * a.piece : start) + a.piece - 1) / a.piece;
    const float *src[MAPS];
    float m[MAPS], inv[MAPS];
#pragma unroll
    for (int x = 0; x < MAPS; x++) {
        src[x] = a.partial + ((((size_t)seq * a.p.heads + h) * MAPS + x) * a.pieces + skip) * (vd + 2);
        m[x] = -INFINITY;
        for (int i = threadIdx.x; i < n; i += 64) m[x] = fmaxf(m[x], src[x][(size_t)i * (vd + 2)]);
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) m[x] = fmaxf(m[x], __shfl_xor(m[x], off, 64));
        float l = 0.f;
        for (int i = 0; i < n; i++) l += src[x][(size_t)i * (vd + 2) + 1] * __builtin_amdgcn_exp2f(src[x][(size_t)i * (vd + 2)] - m[x]);
        inv[x] = (MAPS == 1 ? a.p.out_scale : x == 0 ? 1.0f : -a.p.diff_lambda) / (l + sink_term(a.p, h * MAPS + x, m[x]));
    }
    const auto value = [&](int d) {
        float t = 0.f;
#pragma unroll
        for (int x = 0; x < MAPS; x++) {
            float o = 0.f;
#pragma unroll 4
            for (int i = 0; i < n; i++)
                o = fmaf(src[x][(size_t)i * (vd + 2) + 2 + d], __builtin_amdgcn_exp2f(src[x][(size_t)i * (vd + 2)] - m[x]), o);
            t = fmaf(o, inv[x], t);
        }
        return t;
    };
    bf16 *out = (bf16 *)a.p.out + (size_t)row * a.p.ldo + h * vd;
    if constexpr (MAPS == 2) {
        float v[4], ss = 0.f;  // (the matrix-core kernels take heads of up to 256)
#pragma unroll
        for (int k = 0; k < 4; k++) {
            v[k] = threadIdx.x + k * 64 < vd ? value(threadIdx.x + k * 64) : 0.f;
            ss = fmaf(v[k], v[k], ss);
        }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        const float f = a.p.diff_scale / sqrtf(ss / (float)vd + a.p.diff_eps);
#pragma unroll
        for (int k = 0; k < 4; k++)
            if (threadIdx.x + k * 64 < vd) out[threadIdx.x + k * 64] = (bf16)(v[k] * f);
    } else {
        for (int d = threadIdx.x; d < vd; d += 64) {
            float o = value(d);
            if (a.p.gate) o *= sigmoid_f((float)((const bf16 *)a.p.gate)[(size_t)row * a.p.ldg + h * vd + d]);
            out[d] = (bf16)o;
        }
    }
}

// Both maps' float32 results [rows][heads][2][v_dim] of the plain kernel -> the heads' results. A workgroup per (head, row).
template <typename T>
__global__ void __launch_bounds__(64) diff_kernel(Args a, const float *both) {
    const int h = blockIdx.x, row = blockIdx.y, vd = a.p.v_dim;
    if (a.p.min_rows > 1) {
        const int seq = a.one_token ? row : seq_of_row(a.cu, a.n_seqs, row);
        if ((a.one_token ? 1 : a.cu[seq + 1] - a.cu[seq]) < a.p.min_rows) return;
    }
    const float *x = both + ((size_t)row * a.p.heads + h) * 2 * vd;
    float ss = 0.f;
    for (int d = threadIdx.x; d < vd; d += 64) {
        const float v = fmaf(-a.p.diff_lambda, x[vd + d], x[d]);
        ss = fmaf(v, v, ss);
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    const float f = a.p.diff_scale / sqrtf(ss / (float)vd + a.p.diff_eps);
    for (int d = threadIdx.x; d < vd; d += 64) ((T *)a.p.out)[(size_t)row * a.p.ldo + h * vd + d] = (T)(fmaf(-a.p.diff_lambda, x[vd + d], x[d]) * f);
}

template <int KD, int VD, int QT, int KS, int MAPS>
void launch_prefill(vx_backend *be, Args a, const vx_ragged *b) {
    a.tile_rows = 64 / KS * (QT / MAPS) / a.group;
    a.tiles = count_items(b, a.tile_rows, a.min_rows);
    const size_t lut = a.lut_lds ? (size_t)a.group * a.p.bias_len * 4 : 0;
    const size_t o = KS > 1 ? (size_t)4 / KS * QT * 16 * (VD * 16 + 4) * 4 : 0;
    if (a.tiles > 0) prefill_kernel<KD, VD, QT, KS, MAPS><<<a.tiles * a.p.kv_heads, 256, lut > o ? lut : o, be->stream>>>(a);
}

template <int KD, int VD, int MAPS>
void launch_decode(vx_backend *be, const Args &a, dim3 grid) {
    const size_t lut = a.lut_lds ? (size_t)a.group * a.p.bias_len * 4 : 0, o = (size_t)MAPS * 16 * (VD * 16 + 4) * 4;
    decode_kernel<KD, VD, MAPS><<<grid, 256, lut > o ? lut : o, be->stream>>>(a);
}

template <int KD, int VD, int MAPS = 1>
int run_fast(vx_backend *be, Args a, const vx_ragged *b) {
    bool any_many = false, any_one = !b->q_lens && a.p.min_rows <= 1;
    int64_t many = 0;
    a.min_rows = a.p.min_rows > 2 ? a.p.min_rows : 2;
    if (b->q_lens)
        for (int s = 0; s < b->n_seqs; s++) {
            any_many |= b->q_lens[s] >= a.min_rows, any_one |= b->q_lens[s] == 1 && a.p.min_rows <= 1;
            if (b->q_lens[s] >= a.min_rows) many += b->q_lens[s];
        }
    if (any_many) {
        // Two query tiles a wave halve the keys' traffic; waves that share queries make more workgroups of few rows (the
        // limits are measured). Differential heads: a tile per map.
        const int64_t tiles16 = many * a.p.heads / 16;  // query tiles of the step, per map
        const bool limited = a.p.window > 0 || a.p.chunk > 0;
        const int qt = MAPS == 1 && VD <= 8 && (tiles16 >= 2048 || (tiles16 >= 512 && b->max_kv_len > 1024 && !limited)) ? 2 : 1;
        const int64_t wgs = tiles16 / (4 * qt);
        int ks = wgs >= 384 ? 1 : wgs >= (qt == 2 ? 128 : 256) ? 2 : 4;
        while (ks > 1 && 64 / ks * qt < a.group) ks /= 2;
        if constexpr (VD <= 8 && MAPS == 1) {
            if (qt == 2) {
                if (ks == 1)
                    launch_prefill<KD, VD, 2, 1, 1>(be, a, b);
                else if (ks == 2)
                    launch_prefill<KD, VD, 2, 2, 1>(be, a, b);
                else
                    launch_prefill<KD, VD, 2, 4, 1>(be, a, b);
            }
        }
        if (qt == 1) {
            if (ks == 1)
                launch_prefill<KD, VD, MAPS, 1, MAPS>(be, a, b);
            else if (ks == 2)
                launch_prefill<KD, VD, MAPS, 2, MAPS>(be, a, b);
            else
                launch_prefill<KD, VD, MAPS, 4, MAPS>(be, a, b);
        }
        VX_CHECK_LAUNCH();
    }
    if (any_one) {
        int cu = 256;
        a.piece = 256;
        int span = b->max_kv_len;  // keys of a row, from the start of its first group of 32 on
        if (a.p.window > 0) span = std::min<int64_t>(span, (int64_t)a.p.window + 31);
        if (a.p.chunk > 0) span = std::min<int64_t>(span, (int64_t)a.p.chunk + 31);
        if ((int64_t)b->n_seqs * a.p.kv_heads * ceil_div(span, 256) < 2 * cu) a.piece = 128;
        a.pieces = ceil_div(span, a.piece);
        const size_t bytes = (size_t)b->n_seqs * a.p.heads * MAPS * a.pieces * (a.p.v_dim + 2) * 4;
        int rc = ensure_ws(be, &be->attn_ws, &be->attn_ws_bytes, bytes, "attention");
        if (rc) return rc;
        a.partial = (float *)be->attn_ws;
        be->split.batch = 0;  // (whatever an earlier call left there is gone)
        dim3 grid(a.p.kv_heads, a.pieces, b->n_seqs);
        // vx_pack_batch's list of pieces of 256 tokens, when it was made for this batch
        a.from_start = span == b->max_kv_len;  // (also when windows or chunks start somewhere: they are not much shorter)
        if (a.piece == ATTN_TPW / 2 && a.from_start && be->items.valid && be->items.kv_lens == b->kv_lens && be->items.table_rows == b->table_rows &&
            be->items.batch == b->n_seqs && b->n_seqs * (int64_t)a.pieces <= 65535 &&
            2 * be->items.cap >= (size_t)b->n_seqs * a.pieces) {
            a.items = be->items.buf + (be->items.cap + 1) * 4;
            grid = dim3(a.p.kv_heads, b->n_seqs * a.pieces, 1);
        }
        grid.x *= ceil_div(a.group, 16);
        launch_decode<KD, VD, MAPS>(be, a, grid);
        VX_CHECK_LAUNCH();
        merge_kernel<MAPS><<<dim3(a.p.heads, b->n_seqs), 64, 0, be->stream>>>(a);
        VX_CHECK_LAUNCH();
    }
    return VX_OK;
}

}  // namespace

extern "C" {

size_t vx_kv_block_elems2(int block_size, int k_heads, int k_dim, int v_heads, int v_dim) {
    if (block_size < 1 || k_heads < 1 || k_dim < 1 || v_heads < 1 || v_dim < 1) return 0;
    return (size_t)block_size * ((size_t)k_heads * ((k_dim + 7) & ~7) + (size_t)v_heads * v_dim);
}

size_t vx_kv_block_elems(int block_size, int kv_heads, int k_dim, int v_dim) { return vx_kv_block_elems2(block_size, kv_heads, k_dim, kv_heads, v_dim); }

int vx_attn_ragged_fast(int act, int block_size, int heads, int kv_heads, int k_dim, int v_dim) {
    if (heads < 1 || kv_heads < 1 || heads % kv_heads) return 0;
    const int wide = k_dim > v_dim ? k_dim : v_dim, group = heads / kv_heads;
    return act == VX_ACT_BF16 && block_size == BS && k_dim >= 1 && v_dim >= 1 && wide <= 256 && group <= (wide <= 128 ? 64 : 16);
}

int vx_attn_ragged(vx_backend *be, int act, const vx_ragged *b, const vx_attn_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_attn_ragged");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_attn_ragged: unknown activation type %d", act);
    VX_REQUIRE(p && p->heads >= 1 && p->kv_heads >= 1 && p->heads % p->kv_heads == 0 && p->k_dim >= 1 && p->v_dim >= 1 && p->q &&
                   p->pool && p->out,
               "vx_attn_ragged: bad arguments");
    VX_REQUIRE(p->k_dim <= 2048 && p->v_dim <= 2048, "vx_attn_ragged: heads of %d / %d (at most 2048)", p->k_dim, p->v_dim);
    const int maps = p->maps == 2 ? 2 : 1;
    VX_REQUIRE(p->maps >= 0 && p->maps <= 2 && p->window >= 0 && p->chunk >= 0 && p->softcap >= 0.f, "vx_attn_ragged: bad mask, cap or maps");
    VX_REQUIRE(maps == 1 || (!p->gate && p->out_scale == 1.0f && !p->bias), "vx_attn_ragged: differential heads have no gate, bias or output weight");
    VX_REQUIRE(p->ldq >= p->heads * maps * p->k_dim && p->ldo >= p->heads * p->v_dim && (!p->gate || p->ldg >= p->heads * p->v_dim),
               "vx_attn_ragged: bad strides");
    VX_REQUIRE(!p->bias || p->bias_len >= 1, "vx_attn_ragged: empty bias table");
    VX_REQUIRE(!p->slopes || !p->bias, "vx_attn_ragged: slopes beside a bias table");
    VX_REQUIRE(!p->talk || (maps == 1 && p->softcap == 0.f), "vx_attn_ragged: mixed heads have one map and no cap");
    const bool fast = p->talk ? vx_attn_talk_fast(act, b->block_size, p->heads, p->kv_heads, p->k_dim, p->v_dim)
                              : vx_attn_ragged_fast(act, b->block_size, p->heads, p->kv_heads, p->k_dim, p->v_dim) && (maps == 1 || p->k_dim <= 128);
    VX_REQUIRE(b->rows <= 65535 || fast,
               "vx_attn_ragged: %d rows in one step (at most 65535)", b->rows);
    VX_REQUIRE(b->n_seqs <= 65535, "vx_attn_ragged: %d sequences", b->n_seqs);
    Args a;
    memset(&a, 0, sizeof a);
    a.p = *p;
    if (!a.p.bias) a.p.bias_len = 1;
    a.cu = b->cu_seqlens, a.pos = b->token_pos, a.rows = b->table_rows, a.kv_lens = b->kv_lens, a.tables = b->block_tables;
    a.n_seqs = b->n_seqs, a.max_blocks = b->max_blocks, a.block_size = b->block_size, a.one_token = b->q_lens ? 0 : 1;
    a.kp = (p->k_dim + 7) & ~7;
    a.group = p->heads / p->kv_heads;
    a.vec_q = p->k_dim % 8 == 0 && p->ldq % 8 == 0 && (uintptr_t)p->q % 16 == 0;
    a.vec_o = p->v_dim % 4 == 0 && p->ldo % 4 == 0 && (uintptr_t)p->out % 8 == 0 &&
              (!p->gate || (p->ldg % 4 == 0 && (uintptr_t)p->gate % 8 == 0));
    a.lut_lds = p->bias && (int64_t)a.group * p->bias_len <= LUT_LDS ? 1 : 0;
    if (fast && p->talk) return attn_talk(be, a, b);
    if (fast) {
        const int wide = p->k_dim > p->v_dim ? p->k_dim : p->v_dim;
        if (maps == 2) {
            if (wide <= 64) return run_fast<2, 4, 2>(be, a, b);
            if (p->k_dim <= 64 && p->v_dim <= 128) return run_fast<2, 8, 2>(be, a, b);
            if (wide <= 128) return run_fast<4, 8, 2>(be, a, b);
            return run_fast<4, 16, 2>(be, a, b);
        }
        if (wide <= 64) return run_fast<2, 4>(be, a, b);
        if (wide <= 96) return run_fast<3, 6>(be, a, b);
        if (wide <= 128) return run_fast<4, 8>(be, a, b);
        if (p->k_dim <= 192 && p->v_dim <= 128) return run_fast<6, 8>(be, a, b);
        if (wide <= 192) return run_fast<6, 12>(be, a, b);
        return run_fast<8, 16>(be, a, b);
    }
    PlainAttn t;
    memset(&t, 0, sizeof t);
    t.heads = p->heads * maps, t.group = a.group, t.maps = maps;
    t.q[0] = {p->q, p->ldq, p->k_dim, 0, p->k_dim, p->k_dim};  // (elements, first, room, stride)
    t.row = p->k_dim, t.v_dim = p->v_dim;
    t.pool = p->pool, t.block = (int64_t)vx_kv_block_elems2(b->block_size, p->kv_heads * maps, p->k_dim, p->kv_heads, p->v_dim);
    t.k_head = (int64_t)b->block_size * a.kp, t.k_tok = a.kp;
    t.v_first = p->kv_heads * maps * t.k_head, t.v_head = (int64_t)b->block_size * p->v_dim, t.v_tok = 1, t.v_elem = b->block_size;
    t.scale = p->scale, t.temp_coef = p->temp_coef, t.temp_every = p->temp_every;
    t.bias = p->bias, t.bias_len = p->bias_len, t.sink = p->sink, t.slopes = p->slopes, t.talk = (const bf16 *)p->talk;
    VX_REQUIRE(!p->talk || (int64_t)p->kv_heads * p->k_dim <= 15360, "vx_attn_ragged: %d key heads of %d with mixed heads", p->kv_heads, p->k_dim);
    t.gate = p->gate, t.ldg = p->ldg, t.out_scale = p->out_scale, t.out = p->out, t.ldo = p->ldo, t.out_head = p->v_dim, t.out_cols = p->v_dim;
    t.min_rows = p->min_rows;
    t.window = p->window, t.chunk = p->chunk, t.softcap = p->softcap;
    if (maps == 1) {
        launch_plain(be, act, b, t);
        VX_CHECK_LAUNCH();
        return VX_OK;
    }
    rc = ensure_ws(be, &be->attn_ws, &be->attn_ws_bytes, (size_t)b->rows * p->heads * 2 * p->v_dim * 4, "attention");
    if (rc) return rc;
    be->split.batch = 0;  // (whatever an earlier call left there is gone)
    t.out = be->attn_ws, t.ldo = p->heads * 2 * p->v_dim, t.out_f32 = 1;
    launch_plain(be, act, b, t);
    VX_CHECK_LAUNCH();
    if (act == VX_ACT_BF16)
        diff_kernel<bf16><<<dim3(p->heads, b->rows), 64, 0, be->stream>>>(a, (const float *)be->attn_ws);
    else
        diff_kernel<float><<<dim3(p->heads, b->rows), 64, 0, be->stream>>>(a, (const float *)be->attn_ws);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
