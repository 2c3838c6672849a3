// Shared pieces of the mixed-batch kernels (linear.hip, mixers.hip, attn_ragged.hip, attn_latent.hip): activation types, eight-element
// vectors of them, the matrix-core product of one 16 x 16 x 32 tile, and the map from work items to sequences.
#pragma once

#include "common.h"

namespace vx {

typedef __bf16 bf16;
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x8 __attribute__((ext_vector_type(8)));

template <typename T> struct Vec8;
template <> struct Vec8<bf16> { typedef bf16x8 type; };
template <> struct Vec8<float> { typedef f32x8 type; };
template <typename T> struct Vec4;
template <> struct Vec4<bf16> { typedef bf16x4 type; };
template <> struct Vec4<float> { typedef f32x4 type; };

// acc += A (16 x 32) * B (32 x 16): lane l holds A[l % 16][8 (l / 16) + j] and B[8 (l / 16) + j][l % 16], and of the result
// column l % 16, rows 4 (l / 16) + r.
__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma(bf16x8 a, f32x8 b, f32x4 acc) {  // bfloat16 weights, float32 activations: float32 products
#pragma unroll
    for (int j = 0; j < 8; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32((float)a[j], b[j], acc, 0, 0, 0);
    return acc;
}
// The same product with the activations as A and the weights as B.
__device__ __forceinline__ f32x4 mma_act(bf16x8 a, bf16x8 b, f32x4 acc) { return mma(a, b, acc); }
__device__ __forceinline__ f32x4 mma_act(f32x8 a, bf16x8 b, f32x4 acc) {
#pragma unroll
    for (int j = 0; j < 8; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], (float)b[j], acc, 0, 0, 0);
    return acc;
}

// The wave's number as a scalar: matrix products take no account of lanes that a condition leaves out, so such conditions have to be
// branches of the whole wave.
__device__ __forceinline__ int wave_id() { return __builtin_amdgcn_readfirstlane(threadIdx.x >> 6); }

// The hardware's exponential and reciprocal are good to a unit in the last place; the exponent's own rounding adds |z| times
// that.
__device__ __forceinline__ float sigmoid_f(float z) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.4426950408889634f));
}
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }

// log(1 + exp(z)) = max(z, 0) + log(1 + e), e = exp(-|z|); log(1 + e) = 2 artanh(s), s = e / (2 + e) <= 1/3, by its series
// (the first term left out is below 2e-8 of the sum), which keeps the relative precision of small results.
__device__ __forceinline__ float softplus_f(float z) {
    const float e = expf(-fabsf(z)), s = e / (2.0f + e), q = s * s;
    float t = 1.0f / 13.0f;
    t = fmaf(t, q, 1.0f / 11.0f);
    t = fmaf(t, q, 1.0f / 9.0f);
    t = fmaf(t, q, 1.0f / 7.0f);
    t = fmaf(t, q, 1.0f / 5.0f);
    t = fmaf(t, q, 1.0f / 3.0f);
    return fmaxf(z, 0.f) + 2.0f * fmaf(s * q, t, s);
}

__device__ __forceinline__ void store4(float *p, f32x4 v) { *(f32x4 *)p = v; }
__device__ __forceinline__ void store4(bf16 *p, f32x4 v) {
    bf16x4 o;
#pragma unroll
    for (int i = 0; i < 4; i++) o[i] = (bf16)v[i];
    *(bf16x4 *)p = o;
}

// The sequence a row belongs to: the last one whose first row is not beyond it.
__device__ __forceinline__ int seq_of_row(const int32_t *cu, int n_seqs, int row) {
    int lo = 0, hi = n_seqs - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (cu[mid] <= row)
            lo = mid;
        else
            hi = mid - 1;
    }
    return lo;
}

// Work item `id` of a launch that gives every sequence with at least `min_rows` rows ceil(rows / per_item) items, in
// batch order: its sequence, its index in the sequence and the sequence's item count. False beyond the last. A row may be `each`
// units of which an item takes per_item; max_rows > 0 leaves out sequences with more.
__device__ __forceinline__ bool item_of_seq(const int32_t *cu, int n_seqs, int per_item, int min_rows, int id, int *seq, int *index,
                                            int *count, int each = 1, int max_rows = 0) {
    int c0 = cu[0];
    for (int s = 0; s < n_seqs; s++) {
        const int c1 = cu[s + 1], n = c1 - c0;
        const int items = n < min_rows || (max_rows > 0 && n > max_rows) ? 0 : (n * each + per_item - 1) / per_item;
        if (id < items) {
            *seq = s, *index = id, *count = items;
            return true;
        }
        id -= items;
        c0 = c1;
    }
    return false;
}
// The same count on the host.
inline int count_items(const vx_ragged *b, int per_item, int min_rows) {
    if (!b->q_lens) return min_rows <= 1 ? b->n_seqs : 0;
    int64_t t = 0;
    for (int s = 0; s < b->n_seqs; s++)
        if (b->q_lens[s] >= min_rows) t += ceil_div(b->q_lens[s], per_item);
    return (int)t;
}

// Whether the batch description is complete and its row counts agree.
int check_ragged(const vx_ragged *b, const char *who);

}  // namespace vx
