// What stands at either end of mixed-batch attention: token embeddings with a table of pairs (vx_pair_embedding), and query, key
// and value heads on their way from a float32 projection to the queries' rows and the paged pool (vx_heads_store).
#include "ragged.h"

using namespace vx;

namespace {

struct PairArgs {
    vx_pair_embedding_args p;
    const int32_t *cu, *pos, *slot_map, *table_rows, *tables;
    int n_seqs, max_blocks, block_size, one_token;
};

// A row per workgroup. The token before a sequence's first new row was written by an earlier step.
template <bool VEC>
__global__ void __launch_bounds__(256) pair_embedding_kernel(PairArgs a) {
    const vx_pair_embedding_args &p = a.p;
    const int row = blockIdx.x, pos = a.pos[row], tok = p.tokens[row];
    const int seq = a.one_token ? row : seq_of_row(a.cu, a.n_seqs, row);
    int pair = p.buckets;
    if (pos > 0) {
        int prev;
        if (!a.one_token && row > a.cu[seq]) {
            prev = p.tokens[row - 1];
        } else {
            const int at = pos - 1, blk = a.tables[(size_t)a.table_rows[seq] * a.max_blocks + at / a.block_size];
            prev = p.token_pool[(size_t)blk * a.block_size + at % a.block_size];
        }
        pair = (int)(((int64_t)prev * p.mul_prev + (int64_t)tok * p.mul_cur) % p.buckets);
    }
    if (threadIdx.x == 0) p.token_pool[a.slot_map[row]] = tok;
    const float *e = p.embed + (size_t)tok * p.cols, *b = p.pairs + (size_t)pair * p.cols;
    float *out = p.out + (size_t)row * p.cols;
    if constexpr (VEC) {
        for (int c = threadIdx.x * 4; c < p.cols; c += 1024) *(f32x4 *)(out + c) = *(const f32x4 *)(e + c) + *(const f32x4 *)(b + c);
    } else {
        for (int c = threadIdx.x; c < p.cols; c += 256) out[c] = e[c] + b[c];
    }
}

struct HeadArgs {
    vx_heads_args p;
    const int32_t *slot_map;
    int rows, block_size, units;
};

// A wave takes one head of one row; 64 * NV >= its dimensions. The element a rotation pairs with is read a second time.
template <typename T, int NV>
__global__ void __launch_bounds__(256) heads_kernel(HeadArgs a) {
    const vx_heads_args &p = a.p;
    const int groups = (a.units + 3) / 4, lane = threadIdx.x & 63;
    const int row = blockIdx.x / groups, unit = blockIdx.x % groups * 4 + (threadIdx.x >> 6);
    if (unit >= a.units) return;  // (nothing is shared between waves)
    const bool is_q = unit < p.q_heads, is_k = !is_q && unit < p.q_heads + p.k_heads;
    const int h = is_q ? unit : is_k ? unit - p.q_heads : unit - p.q_heads - p.k_heads;
    const int dim = is_q || is_k ? p.dim : p.v_dim, col = (is_q ? p.q_col : is_k ? p.k_col : p.v_col) + h * dim;
    const float *y = p.y + (size_t)row * p.ldy + col, *bias = p.bias ? p.bias + col : nullptr;
    const auto raw = [&](int d) {
        float t = y[d];
        for (int s = 1; s < p.y_slices; s++) t += y[(size_t)s * p.y_stride + d];
        return bias ? t + bias[d] : t;
    };
    const int kp = (p.dim + 7) & ~7;
    const int slot = is_q ? 0 : a.slot_map[row], blk = is_q ? 0 : slot / a.block_size, in = slot - blk * a.block_size;
    T *pool = (T *)p.pool + (size_t)blk * a.block_size * ((size_t)p.k_heads * kp + (size_t)p.v_heads * p.v_dim);
    T *vpool = pool + (size_t)p.k_heads * a.block_size * kp + (size_t)h * p.v_dim * a.block_size + in;
    float v[NV];
#pragma unroll
    for (int i = 0; i < NV; i++) v[i] = lane + i * 64 < dim ? raw(lane + i * 64) : 0.f;
    if ((is_k && p.v_col < 0) || (!is_q && !is_k)) {
#pragma unroll
        for (int i = 0; i < NV; i++)
            if (lane + i * 64 < dim) vpool[(size_t)(lane + i * 64) * a.block_size] = (T)v[i];
        if (!is_k) return;
    }
    if (p.rot_pairs > 0) {
        const float *tab = p.rot_tab + (size_t)row * p.rot_pairs * 2;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int d = lane + i * 64;
            if (d < 2 * p.rot_pairs) {
                const bool low = d < p.rot_pairs;
                const int pair = low ? d : d - p.rot_pairs;
                const float o = raw(low ? d + p.rot_pairs : d - p.rot_pairs), c = tab[2 * pair], s = tab[2 * pair + 1];
                v[i] = low ? v[i] * c - o * s : v[i] * c + o * s;
            }
        }
    }
    if (p.norm) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; i++) ss = fmaf(v[i], v[i], ss);
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        const float inv = 1.0f / sqrtf(ss / (float)dim + p.eps);
        const float *w = is_q ? p.w_q : p.w_k;
#pragma unroll
        for (int i = 0; i < NV; i++) v[i] *= w && lane + i * 64 < dim ? inv * w[lane + i * 64] : inv;
    }
    T *out = is_q ? (T *)p.q + (size_t)row * p.ldq + h * dim : pool + ((size_t)h * a.block_size + in) * kp;
#pragma unroll
    for (int i = 0; i < NV; i++)
        if (lane + i * 64 < dim) out[lane + i * 64] = (T)v[i];
}

// The same where everything is a multiple of four: LANES lanes take a head, four neighbouring elements each; 4 * LANES >= its
// dimensions. A rotation's partner is LANES' lane rot_pairs / 4 further on.
template <typename T, int LANES>
__global__ void __launch_bounds__(256) heads4_kernel(HeadArgs a) {
    const vx_heads_args &p = a.p;
    const int64_t id = ((int64_t)blockIdx.x * 256 + threadIdx.x) / LANES;
    const int row_ = (int)(id / a.units), unit = (int)(id - (int64_t)row_ * a.units), d = threadIdx.x % LANES * 4;
    const bool live = row_ < a.rows;  // (all lanes stay for the shuffles)
    const int row = live ? row_ : a.rows - 1;
    const bool is_q = unit < p.q_heads, is_k = !is_q && unit < p.q_heads + p.k_heads;
    const int h = is_q ? unit : is_k ? unit - p.q_heads : unit - p.q_heads - p.k_heads;
    const int dim = is_q || is_k ? p.dim : p.v_dim, col = (is_q ? p.q_col : is_k ? p.k_col : p.v_col) + h * dim;
    const bool in_head = d < dim;
    f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
    if (in_head) {
        const float *y = p.y + (size_t)row * p.ldy + col + d;
        v = *(const f32x4 *)y;
#pragma unroll 4
        for (int s = 1; s < p.y_slices; s++) v += *(const f32x4 *)(y + (size_t)s * p.y_stride);
        if (p.bias) v += *(const f32x4 *)(p.bias + col + d);
    }
    const int kp = (p.dim + 7) & ~7;
    const int slot = is_q ? 0 : a.slot_map[row], blk = is_q ? 0 : slot / a.block_size, in = slot - blk * a.block_size;
    T *pool = (T *)p.pool + (size_t)blk * a.block_size * ((size_t)p.k_heads * kp + (size_t)p.v_heads * p.v_dim);
    if (live && in_head && !is_q && (!is_k || p.v_col < 0)) {
        T *vp = pool + (size_t)p.k_heads * a.block_size * kp + ((size_t)h * p.v_dim + d) * a.block_size + in;
#pragma unroll
        for (int e = 0; e < 4; e++) vp[(size_t)e * a.block_size] = (T)v[e];
    }
    if (p.rot_pairs > 0) {
        const bool low = d < p.rot_pairs, turns = (is_q || is_k) && d < 2 * p.rot_pairs;
        const int other = (threadIdx.x & 63) + (turns ? (low ? p.rot_pairs : -p.rot_pairs) / 4 : 0);
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = __shfl(v[e], other, 64);
        if (turns) {
            const float *tab = p.rot_tab + ((size_t)row * p.rot_pairs + (low ? d : d - p.rot_pairs)) * 2;
            const f32x4 t0 = *(const f32x4 *)tab, t1 = *(const f32x4 *)(tab + 4);
            const f32x4 c = f32x4{t0[0], t0[2], t1[0], t1[2]}, s = f32x4{t0[1], t0[3], t1[1], t1[3]};
            v = low ? v * c - o * s : v * c + o * s;
        }
    }
    if (p.norm) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
#pragma unroll
        for (int off = LANES / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        const float inv = 1.0f / sqrtf(ss / (float)dim + p.eps);
        const float *w = is_q ? p.w_q : p.w_k;
        v *= inv;
        if (w && in_head && (is_q || is_k)) v *= *(const f32x4 *)(w + d);
    }
    if (live && in_head && (is_q || is_k)) store4((is_q ? (T *)p.q + (size_t)row * p.ldq + h * dim : pool + ((size_t)h * a.block_size + in) * kp) + d, v);
}

// Norms over all heads of a row: a workgroup takes a row's queries, its keys or its values (blockIdx.y), in pieces of VEC columns; up to
// NV pieces of a thread stay in registers, wider rows are read again.
template <typename T, int VEC, int NV>
__global__ void __launch_bounds__(1024) rows_kernel(HeadArgs a) {
    typedef float F __attribute__((ext_vector_type(VEC)));
    __shared__ float sm[16];
    const vx_heads_args &p = a.p;
    const int row = blockIdx.x, part = blockIdx.y, tid = threadIdx.x, nt = blockDim.x;  // 0: queries, 1: keys, 2: values
    const int dim = part < 2 ? p.dim : p.v_dim, cols = (part == 0 ? p.q_heads : part == 1 ? p.k_heads : p.v_heads) * dim;
    const int col = part == 0 ? p.q_col : part == 1 ? p.k_col : p.v_col;
    const float *y = p.y + (size_t)row * p.ldy + col, *bias = p.bias ? p.bias + col : nullptr, *w = part == 0 ? p.w_q : part == 1 ? p.w_k : nullptr;
    const auto raw = [&](int c) {
        F t = *(const F *)(y + c);
#pragma unroll 4
        for (int s = 1; s < p.y_slices; s++) t += *(const F *)(y + (size_t)s * p.y_stride + c);
        return bias ? t + *(const F *)(bias + c) : t;
    };
    F v[NV];
    float inv = 1.0f, ss = 0.f;
    const auto square = [&](F t) {
#pragma unroll
        for (int e = 0; e < VEC; e++) ss = fmaf(t[e], t[e], ss);
    };
#pragma unroll
    for (int i = 0; i < NV; i++)
        if (const int c = (tid + i * nt) * VEC; c < cols) {
            v[i] = raw(c);
            square(v[i]);
        }
    if (part < 2) {
        for (int c = (tid + NV * nt) * VEC; c < cols; c += nt * VEC) square(raw(c));
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        if ((tid & 63) == 0) sm[tid >> 6] = ss;
        __syncthreads();
        ss = 0.f;
        for (int i = 0; i < (nt >> 6); i++) ss += sm[i];
        inv = 1.0f / sqrtf(ss / (float)cols + p.eps);
    }
    const int kp = (p.dim + 7) & ~7;
    const int slot = part == 0 ? 0 : a.slot_map[row], blk = part == 0 ? 0 : slot / a.block_size, in = slot - blk * a.block_size;
    T *pool = (T *)p.pool + (size_t)blk * a.block_size * ((size_t)p.k_heads * kp + (size_t)p.v_heads * p.v_dim);
    T *vpool = pool + (size_t)p.k_heads * a.block_size * kp + in;
    const auto put = [&](int c, F t) {
        if (part == 2) {
#pragma unroll
            for (int e = 0; e < VEC; e++) vpool[(size_t)(c + e) * a.block_size] = (T)t[e];
            return;
        }
        t *= inv;
        if (w) t *= *(const F *)(w + c);
        T *out = part == 0 ? (T *)p.q + (size_t)row * p.ldq + c : pool + ((size_t)(c / dim) * a.block_size + in) * kp + c % dim;
        if constexpr (VEC == 4) {
            store4(out, t);
        } else {
            out[0] = (T)t[0];
        }
    };
#pragma unroll
    for (int i = 0; i < NV; i++)
        if (const int c = (tid + i * nt) * VEC; c < cols) put(c, v[i]);
    for (int c = (tid + NV * nt) * VEC; c < cols; c += nt * VEC) put(c, raw(c));
}

template <typename T>
void launch_rows(vx_backend *be, const HeadArgs &a) {
    const vx_heads_args &p = a.p;
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = p.dim % 4 == 0 && p.v_dim % 4 == 0 && p.ldy % 4 == 0 && p.q_col % 4 == 0 && p.k_col % 4 == 0 && p.v_col % 4 == 0 && p.ldq % 4 == 0 &&
                     (p.y_slices == 1 || p.y_stride % 4 == 0) && al(p.y) && al(p.bias) && al(p.w_q) && al(p.w_k) && al(p.q) && al(p.pool);
    const dim3 grid(a.rows, p.k_heads > 0 ? 3 : 1);
    int threads = a.rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads * 2 >= p.q_heads * p.dim) threads /= 2;
    if (vec)
        rows_kernel<T, 4, 4><<<grid, threads, 0, be->stream>>>(a);
    else
        rows_kernel<T, 1, 4><<<grid, threads, 0, be->stream>>>(a);
}

template <typename T, int LANES>
void launch_heads4(vx_backend *be, const HeadArgs &a) {
    heads4_kernel<T, LANES><<<(unsigned)ceil_div64((int64_t)a.rows * a.units * LANES, 256), 256, 0, be->stream>>>(a);
}

template <typename T>
void launch_heads(vx_backend *be, const HeadArgs &a) {
    const vx_heads_args &p = a.p;
    if (p.norm == 2) return launch_rows<T>(be, a);
    const int wide = a.p.dim > a.p.v_dim ? a.p.dim : a.p.v_dim;
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    if (p.dim % 4 == 0 && p.v_dim % 4 == 0 && p.ldy % 4 == 0 && p.q_col % 4 == 0 && p.k_col % 4 == 0 && (p.v_col < 0 || p.v_col % 4 == 0) &&
        p.rot_pairs % 4 == 0 && p.ldq % 4 == 0 && (p.y_slices == 1 || p.y_stride % 4 == 0) && al(p.y) && al(p.bias) && al(p.rot_tab) && al(p.w_q) &&
        al(p.w_k) && al(p.q) && al(p.pool) && wide <= 256) {
        if (wide <= 64)
            launch_heads4<T, 16>(be, a);
        else if (wide <= 128)
            launch_heads4<T, 32>(be, a);
        else
            launch_heads4<T, 64>(be, a);
        return;
    }
    const unsigned grid = (unsigned)a.rows * (unsigned)ceil_div(a.units, 4);
    if (wide <= 64)
        heads_kernel<T, 1><<<grid, 256, 0, be->stream>>>(a);
    else if (wide <= 128)
        heads_kernel<T, 2><<<grid, 256, 0, be->stream>>>(a);
    else if (wide <= 256)
        heads_kernel<T, 4><<<grid, 256, 0, be->stream>>>(a);
    else
        heads_kernel<T, 32><<<grid, 256, 0, be->stream>>>(a);
}

}  // namespace

extern "C" {

int vx_pair_embedding(vx_backend *be, const vx_ragged *b, const vx_pair_embedding_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_pair_embedding");
    if (rc) return rc;
    VX_REQUIRE(p && p->cols >= 1 && p->vocab >= 1 && p->buckets >= 1 && p->mul_prev >= 0 && p->mul_cur >= 0 && p->tokens && p->embed && p->pairs &&
                   p->token_pool && p->out,
               "vx_pair_embedding: bad arguments");
    VX_REQUIRE(p->mul_prev < ((int64_t)1 << 31) && p->mul_cur < ((int64_t)1 << 31), "vx_pair_embedding: factors of 2^31 or more");
    const PairArgs a{*p, b->cu_seqlens, b->token_pos, b->slot_mapping, b->table_rows, b->block_tables, b->n_seqs, b->max_blocks, b->block_size,
                     b->q_lens ? 0 : 1};
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    if (p->cols % 4 == 0 && al(p->embed) && al(p->pairs) && al(p->out))
        pair_embedding_kernel<true><<<b->rows, 256, 0, be->stream>>>(a);
    else
        pair_embedding_kernel<false><<<b->rows, 256, 0, be->stream>>>(a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_heads_store(vx_backend *be, int act, const vx_ragged *b, const vx_heads_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_heads_store");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_heads_store: unknown activation type %d", act);
    VX_REQUIRE(p && p->q_heads >= 1 && p->k_heads >= 0 && p->v_heads >= 0 && (p->k_heads > 0) == (p->v_heads > 0) && p->dim >= 1 && p->v_dim >= 1 && p->dim <= 2048 && p->v_dim <= 2048 && p->y &&
                   p->y_slices >= 1 && p->q && (p->pool || p->k_heads == 0) && p->q_col >= 0 && p->k_col >= 0,
               "vx_heads_store: bad arguments");
    VX_REQUIRE(p->v_col >= 0 || (p->v_heads == p->k_heads && p->v_dim == p->dim), "vx_heads_store: values are keys of another size");
    const int64_t q_end = p->q_col + (int64_t)p->q_heads * p->dim, k_end = p->k_col + (int64_t)p->k_heads * p->dim;
    VX_REQUIRE(q_end <= p->ldy && k_end <= p->ldy && (p->v_col < 0 || p->v_col + (int64_t)p->v_heads * p->v_dim <= p->ldy) &&
                   p->ldq >= (int64_t)p->q_heads * p->dim,
               "vx_heads_store: heads beyond their row");
    VX_REQUIRE(p->norm >= 0 && p->norm <= 2 && (p->norm < 2 || (p->rot_pairs == 0 && p->v_col >= 0)), "vx_heads_store: norm %d", p->norm);
    VX_REQUIRE(p->rot_pairs >= 0 && 2 * p->rot_pairs <= p->dim && (p->rot_pairs == 0 || p->rot_tab), "vx_heads_store: %d pairs in heads of %d", p->rot_pairs,
               p->dim);
    HeadArgs a{*p, b->slot_mapping, b->rows, b->block_size, p->q_heads + p->k_heads + (p->v_col < 0 ? 0 : p->v_heads)};
    VX_REQUIRE((int64_t)b->rows * a.units < ((int64_t)1 << 31), "vx_heads_store: %d rows of %d heads", b->rows, a.units);
    if (act == VX_ACT_BF16)
        launch_heads<bf16>(be, a);
    else
        launch_heads<float>(be, a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
