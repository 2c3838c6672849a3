// Tiles of paged attention on the bfloat16 matrix cores, shared by attn_ragged.hip and attn_talk.hip: a wave's keys and values of a
// group of 32, and the running softmax and output of its queries.
//
// Products: S^T = K Q^T and O^T = V^T P^T. The keys of a group are dealt to the two 16-row tiles of S^T so that a lane ends with eight
// consecutive keys of one query, which is the operand layout of the second product; V lies transposed in the pool, so that its operand
// is eight consecutive keys of one dimension as well. The weights P are float32 and enter the second product as two bfloat16 parts
// (16 bits of the 24). Scores, bias, softmax and sums are float32.
#pragma once

#include "attn_plain.h"

namespace vx {

constexpr int BS = 16;               // tokens of a block (matrix-core kernels)
constexpr int LUT_LDS = 12 * 1024;   // floats of bias tables kept in LDS

struct AttnArgs {
    vx_attn_args p;
    const int32_t *cu, *pos, *rows, *kv_lens, *tables;
    int n_seqs, max_blocks, block_size, one_token;
    int kp;            // k_dim up to a multiple of 8
    int group;         // query heads per K/V head
    int vec_q, vec_o;  // vector access to q / gate and out
    int lut_lds;
    // prefill
    int tile_rows, tiles, min_rows;
    // decode
    const int32_t *items;
    int piece, pieces;
    int from_start;    // pieces count from the sequence's start (else from the group of 32 that holds the first key seen)
    float *partial;
};

// The first key a row sees.
__device__ __forceinline__ int first_key(const vx_attn_args &p, int pos) { return first_visible(p.window, p.chunk, pos); }
__device__ __forceinline__ float temperature(const vx_attn_args &p, int pos) {
    return query_temperature(p.temp_coef, p.temp_every, pos);
}
// What the sink adds to a denominator whose terms are relative to m (base-2 exponents). h: head * maps + map.
__device__ __forceinline__ float sink_term(const vx_attn_args &p, int h, float m) {
    return p.sink ? __builtin_amdgcn_exp2f(p.sink[h] * kLog2e - m) : 0.f;
}

__device__ __forceinline__ bf16x8 zero8() {
    bf16x8 z;
#pragma unroll
    for (int i = 0; i < 8; i++) z[i] = (bf16)0.f;
    return z;
}

__device__ __forceinline__ bf16x8 load_q(const bf16 *q, int d, int dim, bool vec) {
    if (vec) return d < dim ? *(const bf16x8 *)(q + d) : zero8();
    bf16x8 v = zero8();
#pragma unroll
    for (int i = 0; i < 8; i++)
        if (d + i < dim) v[i] = q[d + i];
    return v;
}

template <bool NT> __device__ __forceinline__ bf16x8 ld8(const bf16 *p) {
    return NT ? __builtin_nontemporal_load((const bf16x8 *)p) : *(const bf16x8 *)p;
}

// The largest of the four lanes with the same lane % 16. (The copies are opaque: of two equal operands the compiler takes both results for
// equal as well.)
__device__ __forceinline__ float max_of_quarters(float v) {
    typedef unsigned u32x2 __attribute__((ext_vector_type(2)));
    unsigned a = __builtin_bit_cast(unsigned, v), b = a;
    asm("" : "+v"(b));
    u32x2 p = __builtin_bit_cast(u32x2, __builtin_amdgcn_permlane16_swap(a, b, false, false));  // lanes 16 apart
    a = b = __builtin_bit_cast(unsigned, fmaxf(__builtin_bit_cast(float, (unsigned)p[0]), __builtin_bit_cast(float, (unsigned)p[1])));
    asm("" : "+v"(b));
    p = __builtin_bit_cast(u32x2, __builtin_amdgcn_permlane32_swap(a, b, false, false));        // lanes 32 apart
    return fmaxf(__builtin_bit_cast(float, (unsigned)p[0]), __builtin_bit_cast(float, (unsigned)p[1]));
}

// The keys of one group of 32 for a wave: K (of every map) as two 16 x (32 KD) operands, V^T as VD 16 x 32 operands.
template <int KD, int VD, int MAPS, bool NT> struct Keys {
    bf16x8 k[MAPS][2][KD];
    bf16x8 v[VD];
    // lane addresses inside a block
    int ko[2], kd, vo, k_sel, v_sel, kp, v_rows;
    const bf16 *pool;
    size_t blk;
    __device__ __forceinline__ void init(const AttnArgs &a, int g, int lane) {
        const int i = lane & 15, q = lane >> 4;
        pool = (const bf16 *)a.p.pool;
        kp = a.kp, kd = q * 8, v_rows = a.p.v_dim;
        blk = (size_t)a.p.kv_heads * BS * (MAPS * kp + v_rows);
        k_sel = i >> 3, v_sel = q >> 1;
#pragma unroll
        for (int t = 0; t < 2; t++) ko[t] = (g * MAPS * BS + ((i >> 2) & 1) * 8 + t * 4 + (i & 3)) * kp;
        vo = a.p.kv_heads * MAPS * BS * kp + g * v_rows * BS + (q & 1) * 8;
    }
    __device__ __forceinline__ void load_k(int b0, int b1) {
        const bf16 *base = pool + (size_t)(k_sel ? b1 : b0) * blk;
#pragma unroll
        for (int kk = 0; kk < KD; kk++) {
            const int d = kk * 32 + kd;
#pragma unroll
            for (int m = 0; m < MAPS; m++)
#pragma unroll
                for (int t = 0; t < 2; t++) k[m][t][kk] = d < kp ? ld8<NT>(base + m * BS * kp + ko[t] + d) : zero8();
        }
    }
    __device__ __forceinline__ void load_v(int b0, int b1, int lane) {
        const bf16 *base = pool + (size_t)(v_sel ? b1 : b0) * blk + vo;
#pragma unroll
        for (int t = 0; t < VD; t++) v[t] = ld8<NT>(base + min(t * 16 + (lane & 15), v_rows - 1) * BS);
    }
};

// The running softmax and output of QT x 16 queries of a wave.
template <int KD, int VD, int QT> struct Queries {
    bf16x8 q[QT][KD];
    f32x4 o[QT][VD];
    float m[QT], l[QT];       // l: this lane's share of the sum
    float qs[QT], far[QT];    // score factor, bias of the last table entry or slope (for base-2 exponentials)
    int pos[QT], lo[QT], lut[QT];  // position; first key seen; the head's table
    __device__ __forceinline__ void clear() {
#pragma unroll
        for (int t = 0; t < QT; t++) {
            m[t] = -INFINITY, l[t] = 0.f;
#pragma unroll
            for (int v = 0; v < VD; v++) o[t][v] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
    }
    // One group: keys k0 .. k0 + 31. Every key is visible to every query when `whole`; every distance is in the last
    // bias entry when `distant`.
    template <int MAPS, bool NT>
    __device__ __forceinline__ void step(const AttnArgs &a, const Keys<KD, VD, MAPS, NT> &ks, f32x4 st0, f32x4 st1, int t, int k0, int lane, bool whole, bool distant,
                         const float *s_lut) {
        const int key = k0 + (lane >> 4) * 8;
        float s[8];
        if (a.p.softcap > 0.f) {  // cap * tanh(x / cap) = cap * (1 - 2 / (1 + e^(2x / cap))); qs holds 2 / cap, its result stays in base 2
            const float cap = a.p.softcap * kLog2e;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                st0[e] = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(st0[e] * qs[t])), cap);
                st1[e] = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(st1[e] * qs[t])), cap);
            }
        }
        const float factor = a.p.softcap > 0.f ? 1.0f : qs[t];
        if (a.p.slopes) {
            const float b0 = far[t] * (float)(key - pos[t]);
#pragma unroll
            for (int j = 0; j < 8; j++) s[j] = fmaf((j < 4 ? st0[j & 3] : st1[j & 3]), factor, fmaf(far[t], (float)j, b0));
        } else if (distant || !a.p.bias) {
#pragma unroll
            for (int j = 0; j < 8; j++) s[j] = fmaf((j < 4 ? st0[j & 3] : st1[j & 3]), factor, far[t]);
        } else {
            const int last = a.p.bias_len - 1, n0 = pos[t] - key;
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const int n = min(max(n0 - j, 0), last) + lut[t];
                const float b = a.lut_lds ? s_lut[n] : a.p.bias[n] * kLog2e;
                s[j] = fmaf((j < 4 ? st0[j & 3] : st1[j & 3]), factor, b);
            }
        }
        if (!whole) {
#pragma unroll
            for (int j = 0; j < 8; j++)
                if (key + j > pos[t] || key + j < lo[t]) s[j] = -INFINITY;
        }
        float mx = s[0];
#pragma unroll
        for (int j = 1; j < 8; j++) mx = fmaxf(mx, s[j]);
        mx = max_of_quarters(mx);
        const float mn = fmaxf(m[t], mx);
        if (__any(mn > m[t])) {
            const float al = mn > -INFINITY ? __builtin_amdgcn_exp2f(m[t] - mn) : 1.0f;
            l[t] *= al;
#pragma unroll
            for (int v = 0; v < VD; v++) o[t][v] *= al;
            m[t] = mn;
        }
        const float ref = mn > -INFINITY ? mn : 0.f;
        bf16x8 hi, lo;
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const float e = __builtin_amdgcn_exp2f(s[j] - ref);
            l[t] += e;
            hi[j] = (bf16)e;
            lo[j] = (bf16)(e - (float)hi[j]);
        }
#pragma unroll
        for (int v = 0; v < VD; v++) {
            o[t][v] = mma(ks.v[v], hi, o[t][v]);
            o[t][v] = mma(ks.v[v], lo, o[t][v]);
        }
    }
};

__device__ __forceinline__ void write4(const AttnArgs &a, int row, int h, int d, f32x4 v) {
    const vx_attn_args &p = a.p;
    const bf16 *gate = p.gate ? (const bf16 *)p.gate + (size_t)row * p.ldg + h * p.v_dim + d : nullptr;
    bf16 *out = (bf16 *)p.out + (size_t)row * p.ldo + h * p.v_dim + d;
    if (a.vec_o) {  // v_dim is a multiple of 4
        if (d >= p.v_dim) return;
        if (gate) {
            const bf16x4 g4 = *(const bf16x4 *)gate;
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] *= sigmoid_f((float)g4[r]);
        }
        store4(out, v * p.out_scale);
    } else {
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (d + r < p.v_dim) out[r] = (bf16)(v[r] * (gate ? sigmoid_f((float)gate[r]) : 1.0f) * p.out_scale);
    }
}

// Queries::far of head h.
__device__ __forceinline__ float score_offset(const vx_attn_args &p, int h) {
    if (p.slopes) return p.slopes[h] * kLog2e;
    return p.bias ? p.bias[(size_t)h * p.bias_len + p.bias_len - 1] * kLog2e : 0.f;
}

// What a query's scores are multiplied with, for base-2 exponentials or for the cap's exponential.
__device__ __forceinline__ float score_factor(const vx_attn_args &p, int pos) {
    const float f = p.scale * temperature(p, pos) * kLog2e;
    return p.softcap > 0.f ? f * (2.0f / p.softcap) : f;
}

// Attention with scores mixed across heads on the matrix cores (attn_talk.hip), of a geometry that vx_attn_talk_fast takes; a: what
// does not depend on the launch.
int attn_talk(vx_backend *be, AttnArgs a, const vx_ragged *b);

}  // namespace vx
