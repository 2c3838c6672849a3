// Causal attention over a paged pool with nothing tiled: one workgroup per (row, head), any geometry, all in float32 on
// elements of type T. Shared by the kinds of attention; each describes its queries and its pool by strides.
#pragma once

#include "ragged.h"

namespace vx {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int PL_CHUNK = 1024;

// 1 + coef ln(floor((pos + 1) / every) + 1); every 0: 1
__device__ __forceinline__ float query_temperature(float coef, int every, int pos) {
    if (every <= 0) return 1.0f;
    return 1.0f + coef * logf((float)((pos + 1) / every) + 1.0f);
}

// The first key a row sees: all are (0), those of a window of so many tokens, those of its chunk.
__device__ __forceinline__ int first_visible(int window, int chunk, int pos) {
    int f = window > 0 && pos >= window ? pos - window + 1 : 0;
    if (chunk > 0) f = max(f, pos - pos % chunk);
    return f;
}

struct PlainPart {      // one part of a head's query: head h's elements lie at h * stride, and are multiplied with the key row's
    const void *p;      // elements from `first` on; they fill `room` places there, zero beyond n
    int ld, n, first, room, stride;
};

struct PlainAttn {
    int heads, group, row, v_dim;             // row: elements of a key
    PlainPart q[2];
    const void *pool;
    int64_t block, k_head, k_tok, v_first, v_head, v_tok, v_elem;  // strides in elements
    float scale, temp_coef;
    int temp_every;
    const float *bias, *sink, *slopes;
    const bf16 *talk;                         // [heads][heads]: scores are mixed across heads (one map, q[0] alone)
    int bias_len;
    const void *gate;
    int ldg;
    float out_scale;
    void *out;
    int ldo, out_head, out_cols;              // head h at columns h * out_head; columns v_dim .. out_cols - 1 become zero
    int maps, out_f32;                        // maps (0: 1) queries share a head's values; out is float32 whatever T is
    int window, chunk;
    float softcap;
    int min_rows, max_rows;                   // rows of sequences with so many rows only (0: no limit)
    const int32_t *cu, *pos, *rows, *tables;
    int n_seqs, max_blocks, block_size, one_token;
};

template <typename T>
__global__ void __launch_bounds__(256) attn_plain_kernel(PlainAttn p) {
    extern __shared__ float s_q[];  // [row], or with mixed heads [K/V heads][row]
    __shared__ float s_s[PL_CHUNK], s_red[4];
    const int h = blockIdx.x, row = blockIdx.y, maps = max(p.maps, 1), g = h / maps / p.group, tid = threadIdx.x;
    const int seq = p.one_token ? row : seq_of_row(p.cu, p.n_seqs, row);
    const int brings = p.one_token ? 1 : p.cu[seq + 1] - p.cu[seq];
    if ((p.min_rows > 0 && brings < p.min_rows) || (p.max_rows > 0 && brings > p.max_rows)) return;
    const int pos = p.pos[row], len = pos + 1, first = first_visible(p.window, p.chunk, pos);
    const int32_t *bt = p.tables + (size_t)p.rows[seq] * p.max_blocks;
    const T *kpool = (const T *)p.pool + (g * maps + h % maps) * p.k_head;
    const T *vpool = (const T *)p.pool + p.v_first + g * p.v_head;
    const float qf = p.scale * query_temperature(p.temp_coef, p.temp_every, pos);
    // mixed heads: a sum of products with weights is the product with a weighted sum, one for every K/V head
    const int parts = p.talk ? p.heads / p.group : 1;
    if (p.talk) {
        kpool = (const T *)p.pool;
        const bf16 *w = p.talk + (size_t)h * p.heads;
        for (int d = tid; d < parts * p.row; d += 256) {
            const int c = d / p.row, e = d - c * p.row;
            float t = 0.f;
            for (int i = c * p.group; i < (c + 1) * p.group; i++)
                t = fmaf((float)w[i], (float)((const T *)p.q[0].p)[(size_t)row * p.q[0].ld + i * p.q[0].stride + e], t);
            s_q[d] = t;
        }
    }
#pragma unroll
    for (int i = 0; i < 2; i++)
        for (int d = tid; d < p.q[i].room && !p.talk; d += 256)
            s_q[p.q[i].first + d] = d < p.q[i].n ? (float)((const T *)p.q[i].p)[(size_t)row * p.q[i].ld + h * p.q[i].stride + d] : 0.f;
    // thread t accumulates dimension t % width over the keys t / width, t / width + groups, ..; wider heads: several each
    const int width = p.v_dim < 256 ? p.v_dim : 256, kg = 256 / width, md = tid % width, mg = tid / width;
    constexpr int MAXV = 8;  // dimensions of a thread: v_dim <= 2048
    float acc[MAXV];
#pragma unroll
    for (int i = 0; i < MAXV; i++) acc[i] = 0.f;
    float m = -INFINITY, l = 0.f;
    for (int c0 = first; c0 < len; c0 += PL_CHUNK) {
        const int cn = min(PL_CHUNK, len - c0);
        __syncthreads();
        float mx = -INFINITY;
        for (int i = tid; i < cn; i += 256) {
            const int key = c0 + i;
            const T *k = kpool + (size_t)bt[key / p.block_size] * p.block + key % p.block_size * p.k_tok;
            float dot = 0.f;
            for (int c = 0; c < parts; c++)
                for (int d = 0; d < p.row; d++) dot = fmaf(s_q[c * p.row + d], (float)k[c * p.k_head + d], dot);
            float s = dot * qf;
            if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
            if (p.bias) s += p.bias[(size_t)h * p.bias_len + min(pos - key, p.bias_len - 1)];
            if (p.slopes) s -= p.slopes[h] * (float)(pos - key);
            s_s[i] = s;
            mx = fmaxf(mx, s);
        }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
        if ((tid & 63) == 0) s_red[tid >> 6] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(s_red[0], s_red[1]), fmaxf(s_red[2], s_red[3]));
        const float mn = fmaxf(m, mx), al = expf(m - mn);
        float sum = 0.f;
        for (int i = tid; i < cn; i += 256) {
            const float e = expf(s_s[i] - mn);
            s_s[i] = e;
            sum += e;
        }
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
        __syncthreads();
        if ((tid & 63) == 0) s_red[tid >> 6] = sum;
        __syncthreads();
        l = l * al + (s_red[0] + s_red[1] + s_red[2] + s_red[3]);
        m = mn;
        if (mg < kg)
            for (int v = 0; v < MAXV; v++) {
                const int d = md + v * 256;
                if (d >= p.v_dim) break;
                float t = acc[v] * al;
                for (int i = mg; i < cn; i += kg) {
                    const int key = c0 + i;
                    t = fmaf(s_s[i], (float)vpool[(size_t)bt[key / p.block_size] * p.block + d * p.v_elem + key % p.block_size * p.v_tok], t);
                }
                acc[v] = t;
            }
    }
    if (p.sink) l += expf(p.sink[h] - m);
    __syncthreads();
    const size_t at = (size_t)row * p.ldo + h * p.out_head;
    T *out = (T *)p.out + at;
    float *fout = p.out_f32 ? (float *)p.out + at : nullptr;
    float *s_acc = s_s;  // [kg][width]
    for (int v = 0; v < MAXV; v++) {
        const int d = md + v * 256;
        if (v * 256 >= p.v_dim) break;
        if (mg < kg) s_acc[mg * width + md] = acc[v];
        __syncthreads();
        if (mg == 0 && d < p.v_dim) {
            float t = 0.f;
            for (int i = 0; i < kg; i++) t += s_acc[i * width + md];
            t = t / l * p.out_scale;
            if (p.gate) t *= sigmoid_f((float)((const T *)p.gate)[(size_t)row * p.ldg + h * p.v_dim + d]);
            if (fout)
                fout[d] = t;
            else
                out[d] = (T)t;
        }
        __syncthreads();
    }
    for (int d = p.v_dim + tid; d < p.out_cols; d += 256) out[d] = (T)0.f;
}

// t: everything but what the batch says.
inline void launch_plain(vx_backend *be, int act, const vx_ragged *b, PlainAttn t) {
    t.cu = b->cu_seqlens, t.pos = b->token_pos, t.rows = b->table_rows, t.tables = b->block_tables;
    t.n_seqs = b->n_seqs, t.max_blocks = b->max_blocks, t.block_size = b->block_size, t.one_token = b->q_lens ? 0 : 1;
    const dim3 grid(t.heads, b->rows);
    const size_t lds = (size_t)t.row * 4 * (t.talk ? t.heads / t.group : 1);
    if (act == VX_ACT_BF16)
        attn_plain_kernel<bf16><<<grid, 256, lds, be->stream>>>(t);
    else
        attn_plain_kernel<float><<<grid, 256, lds, be->stream>>>(t);
}

}  // namespace vx
