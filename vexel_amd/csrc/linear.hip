// Linear maps with bfloat16 weights for mixed batches (vx_linear_pack, vx_linear), and those of experts over the rows that
// were sorted by expert (vx_linear_experts).
//
// The weights lie in tiles of 16 outputs x 32 inputs, each stored in the order in which the 64 lanes of a wave hold a
// matrix-core operand: a wave reads a tile as one contiguous kilobyte. Both kernels compute W * a^T, so that a lane ends
// with four consecutive output columns of one activation row and stores them together.
//
//  * linear_few_kernel (up to 64 rows: decode steps): bound by the weight stream. A workgroup owns one row tile (two for
//    gate|up pairs), its waves take every WAVES-th step of 32 inputs for all activation rows and meet once, in LDS.
//  * linear_many_kernel (more rows: prompts): tiles of BM rows x BN outputs, four waves in a 2 x 2 grid; the activations go
//    through LDS, double-buffered, the weight operands come straight from memory a step ahead.
//
// Activations are bfloat16 or float32 (template parameter T); with float32 the weights are widened and the float32
// matrix instruction multiplies them, so that nothing is rounded to fewer bits.
#include <string.h>

#include <algorithm>
#include <type_traits>

#include "ragged.h"

using namespace vx;

namespace {

struct LinArgs {
    const void *a;
    const void *w;
    int lda, n, k, rows;
    vx_linear_out o;
    // experts (EX): row0 .. rows - 1 are the places of the workgroup's tile
    int row0;
    const int32_t *tiles;
    int experts, n_shared, k_shared, cols_shared;
    const void *w_shared;
    float shared_limit;
    int common, shared_tiles;  // linear_many_kernel: workgroups for the columns that every tile has, and the shared expert's tiles
};

// The expert and the places of tile `t`; false beyond the last.
__device__ __forceinline__ bool take_tile(LinArgs &p, int t) {
    if (t >= p.tiles[0]) return false;
    const int32_t *r = p.tiles + 4 + 4 * t;
    const int e = r[0];
    p.row0 = r[1], p.rows = r[1] + r[2];
    if (e < p.experts) {
        p.w = (const bf16 *)p.w + (size_t)e * p.n * p.k;
    } else {
        p.w = p.w_shared, p.n = p.n_shared, p.k = p.k_shared, p.o.cols = p.cols_shared, p.o.glu_limit = p.shared_limit;
    }
    return true;
}

// A gate column times its up column.
__device__ __forceinline__ float glu(const vx_linear_out &o, float g, float u) {
    if (o.glu_limit <= 0.f && o.glu_alpha == 0.f) return silu_f(g) * u;
    if (o.glu_limit > 0.f) {
        g = fminf(g, o.glu_limit);
        u = fminf(fmaxf(u, -o.glu_limit), o.glu_limit);
    }
    return g * sigmoid_f(o.glu_alpha * g) * (u + o.glu_add);
}

// One element of a VX_LIN_FORGET map: column c of the activations, or c >= split of the gates.
__device__ __forceinline__ float forget(const vx_linear_out &o, int c, float y) {
    if (c >= o.split) return o.keep[c - o.split] * sigmoid_f(-(y + o.bias[c - o.split]));
    return c < o.silu_cols ? silu_f(y) : y;
}

// Where K and V elements lie in the pool: a part that depends on the slot and one that depends on the column.
struct KvSlot {
    size_t k, v;
};
__device__ __forceinline__ KvSlot kv_slot(const vx_linear_out &o, int row) {
    const int slot = o.slot_mapping ? o.slot_mapping[row] : row, kp = (o.k_dim + 7) & ~7;
    const int blk = slot / o.block_size, in = slot - blk * o.block_size;
    const size_t base = (size_t)blk * o.kv_heads * o.block_size * (kp + o.v_dim);
    return {base + (size_t)in * kp, base + (size_t)o.kv_heads * o.block_size * kp + in};
}
__device__ __forceinline__ int k_used(const vx_linear_out &o) { return o.k_used > 0 ? o.k_used : o.k_dim; }
__device__ __forceinline__ int kv_col_k(const vx_linear_out &o, int ck) {
    const int kp = (o.k_dim + 7) & ~7, g = ck / k_used(o);
    return g * o.block_size * kp + ck - g * k_used(o);
}

// Where row r of the activations lies.
__device__ __forceinline__ size_t a_row(const LinArgs &p, int r) { return p.o.a_rows ? (size_t)p.o.a_rows[r] : (size_t)r; }

template <typename P>
__device__ __forceinline__ void put4(P *row, int c, int cols, int ld, f32x4 v) {
    if (c + 4 <= cols && (ld & 3) == 0) {
        store4(row + c, v);
    } else {
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (c + r < cols) row[c + r] = (P)v[r];
    }
}

// Columns c .. c + 3 of a row, those in the rotated part of their head turned by the row's angles.
__device__ __forceinline__ f32x4 turned(const vx_linear_out &o, int row, int c, f32x4 v) {
    const int pair = (c % o.rot_stride - o.rot_first) >> 1;
    if (c % o.rot_stride < o.rot_first) return v;
    const float *cs = o.rot_tab + ((size_t)row * o.rot_pairs + pair) * 2;
#pragma unroll
    for (int i = 0; i < 2; i++)
        if (pair + i < o.rot_pairs) {
            const float u = v[2 * i], w = v[2 * i + 1], co = cs[2 * i], si = cs[2 * i + 1];
            v[2 * i] = u * co - w * si;
            v[2 * i + 1] = w * co + u * si;
        }
    return v;
}

// The launch's group of independent maps: its weights, its columns of the activations and of the result.
template <typename T>
__device__ __forceinline__ void take_group(LinArgs &p) {
    if (gridDim.z == 1) return;
    const size_t g = blockIdx.z;
    p.w = (const bf16 *)p.w + g * p.n * p.k;
    p.a = (const T *)p.a + g * p.o.a_group;
    p.o.out = p.o.out_f32 ? (void *)((float *)p.o.out + g * p.o.out_group) : (void *)((T *)p.o.out + g * p.o.out_group);
}

// Columns c .. c + 3 of a map with K and V; at: the row's slot, col_k: kv_col_k of the first column where that is K.
template <typename T, int KIND>
__device__ __forceinline__ void emit_kv(const LinArgs &p, KvSlot at, int row, int c, int col_k, f32x4 v) {
    const vx_linear_out &o = p.o;
    const int kw = o.kv_heads * k_used(o), vw = o.kv_heads * o.v_dim, ck = c - o.k_col, cv = c - o.v_col;
    T *pool = (T *)o.pool;
    if (KIND == VX_LIN_KV && ck >= 0 && ck < kw) {
        if ((k_used(o) & 3) == 0 && (o.k_dim & 3) == 0) {
            store4(pool + at.k + col_k, v);
        } else {
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (ck + r < kw) pool[at.k + kv_col_k(o, ck + r)] = (T)v[r];
        }
    } else if (cv >= 0 && cv < vw) {
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (cv + r < vw) pool[at.v + (size_t)(cv + r) * o.block_size] = (T)v[r];
    } else if (KIND == VX_LIN_KV) {
        put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
    }
}

// Columns c .. c + 3 of activation row `row`.
template <typename T, int KIND>
__device__ __forceinline__ void emit(const LinArgs &p, int slice, int row, int c, f32x4 v) {
    const vx_linear_out &o = p.o;
    if (row >= p.rows) return;
    if constexpr (KIND == VX_LIN_PLAIN) {
        if (o.mult != 0.f) v *= o.mult;
        if (o.softcap > 0.f) {
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] = o.softcap * tanhf(v[r] / o.softcap);
        }
        if (o.out_f32)
            put4((float *)o.out + ((size_t)slice * p.rows + row) * o.ldo, c, o.cols, o.ldo, v);
        else
            put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
    } else if constexpr (KIND == VX_LIN_SWIGLU) {
        put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
    } else if constexpr (KIND == VX_LIN_SILU) {
        if (c < o.split) {
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] = silu_f(v[r]);
            put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
        } else {
            put4(o.out2 + (size_t)row * o.ldo2, c - o.split, o.ldo2, o.ldo2, v);
        }
    } else if constexpr (KIND == VX_LIN_FORGET) {
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = forget(o, c + r, v[r]);
        if (c < o.split)
            put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
        else
            put4(o.out2 + (size_t)row * o.ldo2, c - o.split, o.ldo2, o.ldo2, v);
    } else if constexpr (KIND == VX_LIN_RELU2) {
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float t = fmaxf(o.bias && c + r < o.cols ? v[r] + o.bias[c + r] : v[r], 0.f);
            v[r] = t * t;
        }
        put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
    } else if constexpr (KIND == VX_LIN_SPLIT) {
        if (c < o.split)
            put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, v);
        else
            put4(o.out2 + (size_t)row * o.ldo2, c - o.split, o.ldo2, o.ldo2, v);
    } else if constexpr (KIND == VX_LIN_ROTARY) {
        if (c < o.split)
            put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, turned(o, row, c, v));
        else
            put4(o.out2 + (size_t)row * o.ldo2, c - o.split, o.ldo2, o.ldo2, v);
    } else if constexpr (KIND == VX_LIN_SOFTPLUS) {
        f32x4 u;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            u[r] = softplus_f(v[r] + (c + r < o.cols ? o.bias[c + r] : 0.f));
        }
        put4((float *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, u);
    } else {  // VX_LIN_KV, VX_LIN_V: K and V columns leave for the pool (segments start at multiples of 16 columns)
        emit_kv<T, KIND>(p, kv_slot(o, row), row, c, KIND == VX_LIN_KV && c >= o.k_col ? kv_col_k(o, c - o.k_col) : 0, v);
    }
}

// VX_LIN_V, from a tile whose operands were exchanged: rows `row` .. row + 3, column c. Neighbouring slots of a block are
// neighbours in V as it lies in the pool.
template <typename T>
__device__ __forceinline__ void emit_v(const LinArgs &p, const KvSlot *at, bool together, int row, int c, f32x4 v) {
    const vx_linear_out &o = p.o;
    if (row >= p.rows || c >= o.kv_heads * o.v_dim) return;
    T *pool = (T *)o.pool + (size_t)c * o.block_size;
    if (together) {
        store4(pool + at[0].v, v);
    } else {
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (row + r < p.rows) pool[at[r].v] = (T)v[r];
    }
}

// ---------------------------------------------------------------- up to 64 rows
// EX: a workgroup takes one row tile of one expert's map, for all of the expert's rows (grid.z: the experts that have any).
template <typename T, int MT, int NT, int WAVES, int KIND, bool EX>
__global__ void __launch_bounds__(64 * WAVES) linear_few_kernel(LinArgs p) {
    typedef typename Vec8<T>::type A8;
    __shared__ f32x4 red[WAVES][NT * MT][64];
    int mt = MT;  // 16-row tiles that have rows
    if constexpr (EX) {  // (n is a multiple of 32: both of a workgroup's row tiles exist)
        if (!take_tile(p, blockIdx.z) || (int)blockIdx.x * NT >= p.n >> 4) return;
        mt = (p.rows - p.row0 + 15) >> 4;
    } else if constexpr (KIND == VX_LIN_PLAIN) {
        take_group<T>(p);
    }
    const int row0 = EX ? p.row0 : 0;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int steps = p.k >> 5, slices = gridDim.y, slice = blockIdx.y;
    const int s0 = (int)((int64_t)steps * slice / slices), s1 = (int)((int64_t)steps * (slice + 1) / slices);
    const int tile = blockIdx.x * NT;
    const bf16 *w = (const bf16 *)p.w + ((size_t)tile * steps) * 512 + lane * 8;
    const T *a[MT];
#pragma unroll
    for (int m = 0; m < MT; m++) a[m] = (const T *)p.a + a_row(p, min(row0 + m * 16 + (lane & 15), p.rows - 1)) * p.lda + (lane >> 4) * 8;
    f32x4 acc[NT][MT];
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int m = 0; m < MT; m++) acc[t][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int U = sizeof(T) == 4 ? 2 : 4;
    int s = s0 + wave;
    for (; s + (U - 1) * WAVES < s1; s += U * WAVES) {
        bf16x8 wf[U][NT];
        A8 af[U][MT];
#pragma unroll
        for (int u = 0; u < U; u++) {
#pragma unroll
            for (int t = 0; t < NT; t++)
                wf[u][t] = __builtin_nontemporal_load((const bf16x8 *)(w + ((size_t)t * steps + s + u * WAVES) * 512));
#pragma unroll
            for (int m = 0; m < MT; m++)
                if (!EX || m < mt) af[u][m] = *(const A8 *)(a[m] + (size_t)(s + u * WAVES) * 32);
        }
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int t = 0; t < NT; t++)
#pragma unroll
                for (int m = 0; m < MT; m++)
                    if (!EX || m < mt) acc[t][m] = mma(wf[u][t], af[u][m], acc[t][m]);
    }
    for (; s < s1; s += WAVES) {
        bf16x8 wf[NT];
#pragma unroll
        for (int t = 0; t < NT; t++) wf[t] = __builtin_nontemporal_load((const bf16x8 *)(w + ((size_t)t * steps + s) * 512));
#pragma unroll
        for (int m = 0; m < MT; m++) {
            if (EX && m >= mt) break;
            const A8 af = *(const A8 *)(a[m] + (size_t)s * 32);
#pragma unroll
            for (int t = 0; t < NT; t++) acc[t][m] = mma(wf[t], af, acc[t][m]);
        }
    }
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int m = 0; m < MT; m++) red[wave][t * MT + m][lane] = acc[t][m];
    __syncthreads();
    constexpr int ITEMS = (KIND == VX_LIN_SWIGLU ? 1 : NT) * MT * 64;
    for (int i = threadIdx.x; i < ITEMS; i += 64 * WAVES) {
        const int l = i & 63, tm = i >> 6, t = tm / MT, m = tm % MT;
        if (EX && m >= mt) continue;
        f32x4 v = red[0][tm][l];
#pragma unroll
        for (int x = 1; x < WAVES; x++) v += red[x][tm][l];
        const int row = row0 + m * 16 + (l & 15);
        if constexpr (KIND == VX_LIN_SWIGLU) {
            f32x4 u = red[0][MT + m][l];
#pragma unroll
            for (int x = 1; x < WAVES; x++) u += red[x][MT + m][l];
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] = glu(p.o, v[r], u[r]);
            emit<T, KIND>(p, slice, row, (tile / 2) * 16 + (l >> 4) * 4, v);
        } else {
            emit<T, KIND>(p, slice, row, (tile + t) * 16 + (l >> 4) * 4, v);
        }
    }
}

// ---------------------------------------------------------------- more rows
// EX: a row tile is a tile of one expert's places.
template <typename T, int BM, int BN, int KIND, bool EX>
__global__ void __launch_bounds__(256) linear_many_kernel(LinArgs p, int row_tiles) {
    typedef typename Vec8<T>::type A8;
    constexpr int EPC = 16 / (int)sizeof(T);           // elements of a 16-byte piece
    constexpr int CPR = 64 / EPC;                      // pieces of a 64-element row
    constexpr int LOADS = BM * CPR / 256;              // pieces per thread and step
    constexpr int MI = BM / 32, NI = BN / 32;          // 16-wide tiles per wave in each direction
    typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
    extern __shared__ u32x4 lds[];                     // [2][BM][CPR], pieces of a row permuted by the row's low bits
    if constexpr (KIND == VX_LIN_PLAIN && !EX) take_group<T>(p);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int wm = (wave & 1) * (BM / 2), wn = (wave >> 1) * NI;
    // the row tiles of one weight tile run together, with experts on one die (workgroup ids are dealt to the eight dies in turn)
    const int id = EX ? (int)(blockIdx.x & 7) * (int)(gridDim.x >> 3) + (int)(blockIdx.x >> 3) : (int)blockIdx.x;
    int rt = id % row_tiles, nt = id / row_tiles;
    if (EX && id >= p.common) {  // more columns of the shared expert, whose tiles are the last
        if (p.shared_tiles == 0) return;
        const int k = id - p.common;
        rt = p.tiles[0] - p.shared_tiles + k % p.shared_tiles, nt = p.common / row_tiles + k / p.shared_tiles;
    }
    if (EX && (!take_tile(p, rt) || nt * BN >= p.n)) return;
    const int m0 = EX ? p.row0 : rt * BM, tile0 = nt * (BN / 16);
    const int n_tiles = p.n >> 4;
    const int ktiles = p.k >> 6, slices = gridDim.y, slice = blockIdx.y;
    const int k0 = (int)((int64_t)ktiles * slice / slices), k1 = (int)((int64_t)ktiles * (slice + 1) / slices);
    const size_t steps = p.k >> 5;
    auto piece = [](int row, int c) { return row * CPR + (c ^ ((row & 7) * (sizeof(T) == 4 ? 2 : 1))); };

    const bf16 *w[NI];
#pragma unroll
    for (int t = 0; t < NI; t++) w[t] = (const bf16 *)p.w + (size_t)min(tile0 + wn + t, n_tiles - 1) * steps * 512 + lane * 8;
    const u32x4 *ap[LOADS];
    int dst[LOADS];
#pragma unroll
    for (int i = 0; i < LOADS; i++) {
        const int idx = tid + i * 256, row = idx / CPR, c = idx % CPR;
        ap[i] = (const u32x4 *)((const T *)p.a + a_row(p, min(m0 + row, p.rows - 1)) * p.lda) + c;
        dst[i] = piece(row, c);
    }
    u32x4 ar[LOADS];
    bf16x8 wf[2][NI];
    auto fetch = [&](int kt) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) ar[i] = ap[i][(size_t)kt * CPR];
    };
    auto fetch_w = [&](int kt) {
#pragma unroll
        for (int h = 0; h < 2; h++)
#pragma unroll
            for (int t = 0; t < NI; t++) wf[h][t] = *(const bf16x8 *)(w[t] + (size_t)(kt * 2 + h) * 512);
    };
    // V columns alone: the operands are exchanged, so that a lane ends with four rows of one column
    constexpr bool EXCHANGED = KIND == VX_LIN_V;
    f32x4 acc[NI][MI];
#pragma unroll
    for (int t = 0; t < NI; t++)
#pragma unroll
        for (int m = 0; m < MI; m++) acc[t][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (k0 < k1) {
        fetch(k0);
        fetch_w(k0);
    }
    for (int kt = k0; kt < k1; kt++) {
        u32x4 *buf = lds + ((kt - k0) & 1) * BM * CPR;
#pragma unroll
        for (int i = 0; i < LOADS; i++) buf[dst[i]] = ar[i];
        bf16x8 cur[2][NI];
#pragma unroll
        for (int h = 0; h < 2; h++)
#pragma unroll
            for (int t = 0; t < NI; t++) cur[h][t] = wf[h][t];
        __syncthreads();  // (the buffer written now was last read two steps ago, before the barrier of the step between)
        if (kt + 1 < k1) {
            fetch(kt + 1);
            fetch_w(kt + 1);
        }
#pragma unroll
        for (int h = 0; h < 2; h++) {
            A8 af[MI];
#pragma unroll
            for (int m = 0; m < MI; m++) {
                const int row = wm + m * 16 + (lane & 15), q = lane >> 4;
                if constexpr (sizeof(T) == 2) {
                    af[m] = *(const A8 *)(buf + piece(row, h * 4 + q));
                } else {  // (the two pieces of eight floats stay neighbours)
                    af[m] = *(const A8 *)(buf + piece(row, h * 8 + q * 2));
                }
            }
#pragma unroll
            for (int t = 0; t < NI; t++)
#pragma unroll
                for (int m = 0; m < MI; m++) acc[t][m] = EXCHANGED ? mma_act(af[m], cur[h][t], acc[t][m]) : mma(cur[h][t], af[m], acc[t][m]);
        }
    }
    const int q4 = (lane >> 4) * 4;
    if constexpr (EXCHANGED) {
#pragma unroll
        for (int m = 0; m < MI; m++) {
            const int row = m0 + wm + m * 16 + q4;
            KvSlot at[4];
#pragma unroll
            for (int r = 0; r < 4; r++) at[r] = kv_slot(p.o, min(row + r, p.rows - 1));
            const bool together = row + 4 <= p.rows && (p.o.block_size & 3) == 0 && (at[0].v & 3) == 0 && at[1].v == at[0].v + 1 && at[2].v == at[0].v + 2 &&
                                  at[3].v == at[0].v + 3;
#pragma unroll
            for (int t = 0; t < NI; t++)
                if (tile0 + wn + t < n_tiles) emit_v<T>(p, at, together, row, (tile0 + wn + t) * 16 + (lane & 15), acc[t][m]);
        }
        return;
    } else if constexpr (KIND == VX_LIN_KV) {
        int col_k[NI];
#pragma unroll
        for (int t = 0; t < NI; t++) {
            const int ck = (tile0 + wn + t) * 16 + q4 - p.o.k_col;
            col_k[t] = ck >= 0 ? kv_col_k(p.o, ck) : 0;
        }
#pragma unroll
        for (int m = 0; m < MI; m++) {
            const int row = m0 + wm + m * 16 + (lane & 15);
            if (row >= p.rows) continue;
            const KvSlot at = kv_slot(p.o, row);
#pragma unroll
            for (int t = 0; t < NI; t++)
                if (tile0 + wn + t < n_tiles) emit_kv<T, KIND>(p, at, row, (tile0 + wn + t) * 16 + q4, col_k[t], acc[t][m]);
        }
        return;
    }
#pragma unroll
    for (int m = 0; m < MI; m++) {
        const int row = m0 + wm + m * 16 + (lane & 15);
        if constexpr (KIND == VX_LIN_SWIGLU) {
#pragma unroll
            for (int t = 0; t < NI; t += 2) {
                if (tile0 + wn + t >= n_tiles) continue;
                f32x4 v;
#pragma unroll
                for (int r = 0; r < 4; r++) v[r] = glu(p.o, acc[t][m][r], acc[t + 1][m][r]);
                emit<T, KIND>(p, slice, row, (tile0 + wn + t) / 2 * 16 + q4, v);
            }
        } else {
#pragma unroll
            for (int t = 0; t < NI; t++)
                if (tile0 + wn + t < n_tiles) emit<T, KIND>(p, slice, row, (tile0 + wn + t) * 16 + q4, acc[t][m]);
        }
    }
}

// Adds up the slices of a VX_LIN_SPLIT, VX_LIN_ROTARY, VX_LIN_SILU or VX_LIN_FORGET map and deals the columns to its two results.
template <typename T>
__global__ void __launch_bounds__(256) split_sum_kernel(const float *part, int slices, int rows, int n, vx_linear_out o) {
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int per = n / 4, row = (int)(id / per), c = (int)(id % per) * 4;
    if (row >= rows) return;
    const float *src = part + (size_t)row * n + c;
    f32x4 v = *(const f32x4 *)src;
    for (int s = 1; s < slices; s++) v += *(const f32x4 *)(src + (size_t)s * rows * n);
    if (c < o.split && o.kind == VX_LIN_SILU)
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = silu_f(v[r]);
    if (o.kind == VX_LIN_FORGET)
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = forget(o, c + r, v[r]);
    if (c < o.split)
        put4((T *)o.out + (size_t)row * o.ldo, c, o.cols, o.ldo, o.rot_tab ? turned(o, row, c, v) : v);
    else
        put4(o.out2 + (size_t)row * o.ldo2, c - o.split, o.ldo2, o.ldo2, v);
}

// ---------------------------------------------------------------- packing
__global__ void linear_pack_kernel(const uint16_t *src, int n, int k, uint16_t *dst, int k_pad, int tile0, int tile_step, int col0) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * k) return;
    const int r = (int)(i / k), c = (int)(i % k) + col0;
    const int tile = tile0 + (r >> 4) * tile_step, step = c >> 5, lane = (r & 15) + 16 * ((c & 31) >> 3);
    dst[((size_t)tile * (k_pad >> 5) + step) * 512 + lane * 8 + (c & 7)] = src[i];
}

__global__ void fill_zero_kernel(uint32_t *p, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) p[i] = 0;
}

// ---------------------------------------------------------------- launches
template <typename T, int MT, int NT, int WAVES, int KIND>
void launch_few_as(vx_backend *be, const LinArgs &p, int slices) {
    linear_few_kernel<T, MT, NT, WAVES, KIND, false><<<dim3((p.n >> 4) / NT, slices, p.o.groups), 64 * WAVES, 0, be->stream>>>(p);
}
template <typename T, int MT, int KIND>
void launch_few(vx_backend *be, const LinArgs &p, int slices) {
    const int tiles = p.n >> 4;
    // two row tiles to a workgroup (an activation operand serves both) where that leaves enough workgroups
    if constexpr (KIND == VX_LIN_SWIGLU) {
        launch_few_as<T, MT, 2, MT == 4 ? 4 : 8, KIND>(be, p, slices);
    } else if constexpr (MT < 4) {
        if (tiles % 2 == 0 && (int64_t)tiles / 2 * slices * p.o.groups >= 512)
            launch_few_as<T, MT, 2, 8, KIND>(be, p, slices);
        else
            launch_few_as<T, MT, 1, 8, KIND>(be, p, slices);
    } else {
        launch_few_as<T, MT, 1, 8, KIND>(be, p, slices);
    }
}

template <typename T, int BM, int BN, int KIND>
void launch_many(vx_backend *be, const LinArgs &p, int slices) {
    const int rt = ceil_div(p.rows, BM), nt = ceil_div(p.n, BN);
    linear_many_kernel<T, BM, BN, KIND, false><<<dim3(rt * nt, slices, p.o.groups), 256, 2 * BM * 64 * sizeof(T), be->stream>>>(p, rt);
}

// The widest tiles that still give every compute unit a workgroup.
void many_tile(int n, int rows, int slices, int *bm, int *bn) {
    auto wgs = [&](int m, int nn) { return (int64_t)ceil_div(rows, m) * ceil_div(n, nn) * slices; };
    *bm = 128, *bn = 128;
    if (wgs(128, 128) >= 256) return;
    *bm = 64;
    if (wgs(64, 128) >= 256) return;
    *bn = 64;
}

// In how many slices of its inputs a map is best computed, when something adds the slices up afterwards.
int pick_slices(int n, int k, int rows) {
    const int ktiles = k / 64;
    int64_t wgs;
    int want, least;
    if (rows <= 64) {
        wgs = n / 16, want = 1024, least = 4;  // (as many workgroups as the chip holds; a wave's step of 32 inputs)
        if (wgs >= want) return 1;
    } else {
        wgs = (int64_t)ceil_div(rows, 128) * ceil_div(n, 128), want = 512, least = 12;
        if (wgs >= 384) return 1;
    }
    int s = (int)((want + wgs - 1) / wgs);
    if (s > 8) s = 8;
    if (s > ktiles / least) s = ktiles / least;
    return s < 1 ? 1 : s;
}

template <typename T, int KIND>
int launch(vx_backend *be, const LinArgs &p, int slices) {
    if (p.rows <= 64) {
        if (p.rows <= 16)
            launch_few<T, 1, KIND>(be, p, slices);
        else if (p.rows <= 32)
            launch_few<T, 2, KIND>(be, p, slices);
        else
            launch_few<T, 4, KIND>(be, p, slices);
    } else {
        int bm, bn;
        many_tile(p.n, p.rows, slices * p.o.groups, &bm, &bn);
        if constexpr (sizeof(T) == 4) {
            launch_many<T, 64, 64, KIND>(be, p, slices);
        } else if (bn == 64) {
            launch_many<T, 64, 64, KIND>(be, p, slices);
        } else if (bm == 64) {
            launch_many<T, 64, 128, KIND>(be, p, slices);
        } else {
            launch_many<T, 128, 128, KIND>(be, p, slices);
        }
    }
    VX_CHECK_LAUNCH();
    return VX_OK;
}

template <typename T>
int dispatch(vx_backend *be, const LinArgs &p, int slices) {
    switch (p.o.kind) {
        case VX_LIN_PLAIN: return launch<T, VX_LIN_PLAIN>(be, p, slices);
        case VX_LIN_SWIGLU: return launch<T, VX_LIN_SWIGLU>(be, p, slices);
        case VX_LIN_KV: return launch<T, VX_LIN_KV>(be, p, slices);
        case VX_LIN_SPLIT: return launch<T, VX_LIN_SPLIT>(be, p, slices);
        case VX_LIN_ROTARY: return launch<T, VX_LIN_ROTARY>(be, p, slices);
        case VX_LIN_SILU: return launch<T, VX_LIN_SILU>(be, p, slices);
        case VX_LIN_V: return launch<T, VX_LIN_V>(be, p, slices);
        case VX_LIN_FORGET: return launch<T, VX_LIN_FORGET>(be, p, slices);
        case VX_LIN_RELU2: return launch<T, VX_LIN_RELU2>(be, p, slices);
        default: return launch<T, VX_LIN_SOFTPLUS>(be, p, slices);
    }
}

template <typename T, int BM, int BN, int KIND>
void launch_many_experts(vx_backend *be, LinArgs p, int step_rows, int max_tiles) {
    const int nts = ceil_div(p.n, BN), more = p.n_shared > p.n ? ceil_div(p.n_shared, BN) - nts : 0;
    p.common = max_tiles * nts, p.shared_tiles = more > 0 ? ceil_div(step_rows, BM) : 0;
    const int grid = ceil_div(p.common + p.shared_tiles * more, 8) * 8;
    linear_many_kernel<T, BM, BN, KIND, true><<<grid, 256, 2 * BM * 64 * sizeof(T), be->stream>>>(p, max_tiles);
}

// Experts' maps. Up to 64 rows in the step: an expert's rows are one tile, and every active expert's weights are read once.
template <typename T, int KIND>
int launch_experts(vx_backend *be, const LinArgs &p, int step_rows, int max_tiles, int tile_rows) {
    const int n = std::max(p.n, p.n_shared);
    if (step_rows <= 64) {
        constexpr int NT = 2;
        const dim3 grid(ceil_div(n >> 4, NT), 1, max_tiles);
        if (step_rows <= 16)
            linear_few_kernel<T, 1, NT, 8, KIND, true><<<grid, 512, 0, be->stream>>>(p);
        else if (step_rows <= 32)
            linear_few_kernel<T, 2, NT, 8, KIND, true><<<grid, 512, 0, be->stream>>>(p);
        else
            linear_few_kernel<T, 4, NT, 4, KIND, true><<<grid, 256, 0, be->stream>>>(p);
    } else if (sizeof(T) == 2 && tile_rows == 128) {
        if constexpr (sizeof(T) == 2)
            launch_many_experts<T, 128, 128, KIND>(be, p, step_rows, max_tiles);
    } else if constexpr (sizeof(T) == 2) {
        launch_many_experts<T, 64, 128, KIND>(be, p, step_rows, max_tiles);
    } else {
        launch_many_experts<T, 64, 64, KIND>(be, p, step_rows, max_tiles);
    }
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // namespace

namespace vx {
int check_ragged(const vx_ragged *b, const char *who) {
    VX_REQUIRE(b != nullptr, "%s: null batch", who);
    VX_REQUIRE(b->cu_seqlens && b->token_pos && b->slot_mapping && b->table_rows && b->kv_lens && b->block_tables,
               "%s: null batch array", who);
    VX_REQUIRE(b->rows >= 1 && b->n_seqs >= 1 && b->max_blocks >= 1 && b->block_size >= 1 && b->max_kv_len >= 1 &&
                   b->max_kv_len <= (int64_t)b->max_blocks * b->block_size,
               "%s: bad batch sizes", who);
    if (b->q_lens) {
        int64_t t = 0;
        for (int s = 0; s < b->n_seqs; s++) {
            VX_REQUIRE(b->q_lens[s] >= 1, "%s: sequence %d brings no rows", who, s);
            t += b->q_lens[s];
        }
        VX_REQUIRE(t == b->rows, "%s: the sequences bring %lld rows, the batch has %d", who, (long long)t, b->rows);
    } else {
        VX_REQUIRE(b->rows == b->n_seqs, "%s: %d rows for %d sequences of one row", who, b->rows, b->n_seqs);
    }
    return VX_OK;
}
}  // namespace vx

extern "C" {

int vx_fill_zero(vx_backend *be, void *dst, size_t bytes) {
    int rc = enter(be);
    if (rc) return rc;
    if (bytes == 0) return VX_OK;
    VX_REQUIRE(dst && bytes % 4 == 0 && (uintptr_t)dst % 4 == 0, "vx_fill_zero: bad arguments");
    items_written(be, dst, bytes);
    const size_t n = bytes / 4;
    const int grid = (int)(n / 256 + 1 < 4096 ? n / 256 + 1 : 4096);
    fill_zero_kernel<<<grid, 256, 0, be->stream>>>((uint32_t *)dst, n);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

size_t vx_linear_bytes(int n_pad, int k_pad) { return n_pad > 0 && k_pad > 0 ? (size_t)n_pad * k_pad * 2 : 0; }

int vx_linear_pack(vx_backend *be, const void *src, int n, int k, void *dst, int n_pad, int k_pad, int tile0, int tile_step,
                   int col0) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(src && dst && n > 0 && k > 0 && tile0 >= 0 && tile_step >= 1 && col0 >= 0, "vx_linear_pack: bad arguments");
    VX_REQUIRE(n_pad % 16 == 0 && k_pad % 64 == 0 && col0 + k <= k_pad && tile0 + (int64_t)((n - 1) / 16) * tile_step < n_pad / 16,
               "vx_linear_pack: [%d, %d] at tile %d (step %d), column %d does not fit [%d, %d]", n, k, tile0, tile_step, col0, n_pad,
               k_pad);
    linear_pack_kernel<<<(unsigned)ceil_div64((int64_t)n * k, 256), 256, 0, be->stream>>>((const uint16_t *)src, n, k, (uint16_t *)dst,
                                                                                         k_pad, tile0, tile_step, col0);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_linear_slices(vx_backend *be, int n, int k, int rows) {
    (void)be;
    if (n <= 0 || k <= 0 || rows <= 0) return 1;
    return pick_slices(n, k, rows);
}

int vx_linear(vx_backend *be, int act, const void *a, int lda, const void *w, int n, int k, int rows, const vx_linear_out *o) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(a && w && o && o->out && rows >= 1, "vx_linear: bad arguments");
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_linear: unknown activation type %d", act);
    VX_REQUIRE(n >= 16 && n % 16 == 0 && k >= 64 && k % 64 == 0 && lda >= k && lda % 8 == 0 && (uintptr_t)a % 16 == 0 &&
                   (uintptr_t)w % 16 == 0 && (uintptr_t)o->out % 16 == 0,
               "vx_linear: sizes or alignment (n %d, k %d, lda %d)", n, k, lda);
    VX_REQUIRE(o->kind >= VX_LIN_PLAIN && o->kind <= VX_LIN_RELU2, "vx_linear: unknown kind %d", o->kind);
    VX_REQUIRE(o->cols >= 1 && o->ldo >= o->cols, "vx_linear: %d columns in rows of %d", o->cols, o->ldo);
    const int slices = o->slices > 1 ? o->slices : 1;
    VX_REQUIRE(slices == 1 || (o->kind == VX_LIN_PLAIN && o->out_f32 && slices <= 64), "vx_linear: slices need a plain float32 result");
    if (o->kind == VX_LIN_SWIGLU) {
        VX_REQUIRE(n % 32 == 0 && o->cols <= n / 2, "vx_linear: gate|up pairs of %d rows for %d columns", n, o->cols);
        VX_REQUIRE(o->glu_limit >= 0.f, "vx_linear: negative limit");
    } else if (o->kind == VX_LIN_SPLIT || o->kind == VX_LIN_SILU || o->kind == VX_LIN_FORGET) {
        VX_REQUIRE(o->out2 && o->split % 16 == 0 && o->split > 0 && o->split < n && o->cols == o->split && o->ldo2 >= n - o->split &&
                       (uintptr_t)o->out2 % 16 == 0,
                   "vx_linear: bad split");
    } else if (o->kind == VX_LIN_ROTARY) {
        VX_REQUIRE(o->split % 16 == 0 && o->split > 0 && o->split <= n && o->cols == o->split &&
                       (o->split == n || (o->out2 && o->ldo2 >= n - o->split && (uintptr_t)o->out2 % 16 == 0)),
                   "vx_linear: bad split");
        VX_REQUIRE(o->rot_tab && o->rot_pairs >= 1 && o->rot_first >= 0 && o->rot_first % 4 == 0 && o->rot_stride % 4 == 0 &&
                       o->rot_first + 2 * o->rot_pairs <= o->rot_stride,
                   "vx_linear: %d rotated pairs at %d in heads of %d columns", o->rot_pairs, o->rot_first, o->rot_stride);
    } else {
        VX_REQUIRE(o->cols <= n, "vx_linear: %d columns of %d", o->cols, n);
    }
    if (o->kind == VX_LIN_SOFTPLUS || o->kind == VX_LIN_FORGET) VX_REQUIRE(o->bias != nullptr, "vx_linear: null bias");
    if (o->kind == VX_LIN_FORGET) VX_REQUIRE(o->keep && o->silu_cols >= 0 && o->silu_cols <= o->split, "vx_linear: incomplete gates");
    VX_REQUIRE(o->mult == 0.f || (o->kind == VX_LIN_PLAIN && slices == 1), "vx_linear: a factor needs a plain whole result");
    if (o->kind == VX_LIN_KV || o->kind == VX_LIN_V)
        VX_REQUIRE(o->pool && o->kv_heads >= 1 && o->k_dim >= 1 && o->v_dim >= 1 && o->block_size >= 1 &&
                       o->k_col % 16 == 0 && o->v_col % 16 == 0 && o->k_col >= 0 && o->v_col >= 0 &&
                       (o->kind == VX_LIN_V || (o->k_used >= 0 && o->k_used <= o->k_dim && o->k_col + o->kv_heads * (o->k_used > 0 ? o->k_used : o->k_dim) <= n)) &&
                       ((o->kind == VX_LIN_KV && o->v_col == n) || o->v_col + o->kv_heads * o->v_dim <= n),
                   "vx_linear: bad K/V columns");
    if (o->kind == VX_LIN_V) VX_REQUIRE(o->v_col == 0 && o->kv_heads * o->v_dim + 15 >= n, "vx_linear: columns beside V");
    VX_REQUIRE(o->softcap == 0.f || (o->softcap > 0.f && o->kind == VX_LIN_PLAIN && slices == 1), "vx_linear: a cap needs a plain whole result");
    LinArgs p;
    memset(&p, 0, sizeof p);
    p.a = a, p.w = w, p.lda = lda, p.n = n, p.k = k, p.rows = rows, p.o = *o;
    if (o->groups > 1) {
        VX_REQUIRE(o->kind == VX_LIN_PLAIN && slices == 1 && o->groups <= 65535 && o->a_group >= 0 && o->out_group >= o->cols &&
                       o->a_group % 8 == 0 && o->out_group % 4 == 0 && lda >= (o->groups - 1) * (int64_t)o->a_group + k &&
                       o->ldo >= (o->groups - 1) * (int64_t)o->out_group + o->cols,
                   "vx_linear: bad groups");
    } else {
        p.o.groups = 1;
    }
    if (o->kind != VX_LIN_ROTARY) p.o.rot_tab = nullptr;
    if (o->kind == VX_LIN_SPLIT || o->kind == VX_LIN_ROTARY || o->kind == VX_LIN_SILU || o->kind == VX_LIN_FORGET) {  // (narrow and deep as a rule) in slices, added up by a kernel of their own
        const int cut = k >= 2048 ? pick_slices(n, k, rows) : 1;  // (a short map is over before the second launch pays)
        if (cut > 1) {
            const size_t bytes = (size_t)cut * rows * n * 4;
            rc = ensure_ws(be, &be->part_ws, &be->part_ws_bytes, bytes, "partial sums");
            if (rc) return rc;
            p.o.kind = VX_LIN_PLAIN, p.o.out_f32 = 1, p.o.out = be->part_ws, p.o.ldo = p.o.cols = n;
            rc = act == VX_ACT_BF16 ? dispatch<bf16>(be, p, cut) : dispatch<float>(be, p, cut);
            if (rc) return rc;
            const unsigned grid = (unsigned)ceil_div64((int64_t)rows * (n / 4), 256);
            if (act == VX_ACT_BF16)
                split_sum_kernel<bf16><<<grid, 256, 0, be->stream>>>((const float *)be->part_ws, cut, rows, n, *o);
            else
                split_sum_kernel<float><<<grid, 256, 0, be->stream>>>((const float *)be->part_ws, cut, rows, n, *o);
            VX_CHECK_LAUNCH();
            return VX_OK;
        }
    }
    return act == VX_ACT_BF16 ? dispatch<bf16>(be, p, slices) : dispatch<float>(be, p, slices);
}

int vx_route_tile_rows(int act, int rows, int experts, int top) {
    if (rows <= 64 || act != VX_ACT_BF16) return 64;
    return (int64_t)rows * top >= (int64_t)experts * 96 ? 128 : 64;
}

int vx_linear_experts(vx_backend *be, int act, const vx_experts_args *e) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_linear_experts: unknown activation type %d", act);
    VX_REQUIRE(e && e->a && e->w && e->tiles && e->out && e->rows >= 1 && e->experts >= 1 && e->max_tiles >= 1, "vx_linear_experts: bad arguments");
    VX_REQUIRE(e->kind == VX_LIN_PLAIN || e->kind == VX_LIN_SWIGLU || e->kind == VX_LIN_RELU2, "vx_linear_experts: kind %d", e->kind);
    VX_REQUIRE((e->rows <= 64 && e->tile_rows == 64) || (e->rows > 64 && (e->tile_rows == 64 || (e->tile_rows == 128 && act == VX_ACT_BF16))),
               "vx_linear_experts: tiles of %d of %d rows", e->tile_rows, e->rows);
    const int per = e->kind == VX_LIN_SWIGLU ? 2 : 1;  // outputs of a result column
    const auto fits = [&](const void *w, int n, int k, int cols) {
        return w && (uintptr_t)w % 16 == 0 && n >= 32 && n % 32 == 0 && k >= 64 && k % 64 == 0 && e->lda >= k && cols >= 1 && cols * per <= n &&
               cols <= e->ldo;
    };
    VX_REQUIRE(fits(e->w, e->n, e->k, e->cols) && (!e->shared || fits(e->w_shared, e->n_shared, e->k_shared, e->cols_shared)) && e->lda % 8 == 0 &&
                   (uintptr_t)e->a % 16 == 0 && (uintptr_t)e->out % 16 == 0,
               "vx_linear_experts: sizes or alignment (n %d, k %d, lda %d)", e->n, e->k, e->lda);
    VX_REQUIRE(e->glu_limit >= 0.f && e->shared_limit >= 0.f && e->max_tiles <= 65535 * 16, "vx_linear_experts: bad limit or tile count");
    VX_REQUIRE(e->rows > 64 || e->max_tiles <= 65535, "vx_linear_experts: %d tiles", e->max_tiles);
    LinArgs p;
    memset(&p, 0, sizeof p);
    p.a = e->a, p.w = e->w, p.lda = e->lda, p.n = e->n, p.k = e->k;
    p.o.kind = e->kind, p.o.out = e->out, p.o.ldo = e->ldo, p.o.cols = e->cols, p.o.a_rows = e->a_rows, p.o.groups = 1;
    p.o.glu_limit = e->glu_limit, p.o.glu_alpha = e->glu_alpha, p.o.glu_add = e->glu_add;
    p.tiles = e->tiles, p.experts = e->experts;
    if (e->shared) p.w_shared = e->w_shared, p.n_shared = e->n_shared, p.k_shared = e->k_shared, p.cols_shared = e->cols_shared, p.shared_limit = e->shared_limit;
    if (e->kind == VX_LIN_SWIGLU)
        return act == VX_ACT_BF16 ? launch_experts<bf16, VX_LIN_SWIGLU>(be, p, e->rows, e->max_tiles, e->tile_rows)
                                  : launch_experts<float, VX_LIN_SWIGLU>(be, p, e->rows, e->max_tiles, e->tile_rows);
    if (e->kind == VX_LIN_RELU2)
        return act == VX_ACT_BF16 ? launch_experts<bf16, VX_LIN_RELU2>(be, p, e->rows, e->max_tiles, e->tile_rows)
                                  : launch_experts<float, VX_LIN_RELU2>(be, p, e->rows, e->max_tiles, e->tile_rows);
    return act == VX_ACT_BF16 ? launch_experts<bf16, VX_LIN_PLAIN>(be, p, e->rows, e->max_tiles, e->tile_rows)
                              : launch_experts<float, VX_LIN_PLAIN>(be, p, e->rows, e->max_tiles, e->tile_rows);
}

}  // extern "C"
