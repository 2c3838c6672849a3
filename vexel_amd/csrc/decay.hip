// Linear attention with a constant decay per head over mixed batches (vx_decay_attn), and the norm with a gate behind it
// (vx_gated_norm).
//
//  * step_kernel: sequences that bring few rows (and everything in float32 batches). A workgroup keeps 32 columns of one head's
//    state in registers and walks the rows; bound by reading and writing the state.
//  * Sequences with more rows, on the bfloat16 matrix cores, in chunks of one or two sub-chunks of 64 rows:
//      chunk_kernel   what a chunk adds to the state, K^T (decayed) V
//      carry_kernel   runs over the chunks: the state before each of them, and the final one
//      out_kernel     a sub-chunk's rows: Q S with the state before the chunk, and (Q K^T, decayed) V inside the chunk
//    Float32 operands (decayed keys, scores, states) enter the products as two bfloat16 parts (16 bits of the 24). Products whose
//    inner dimension is the token read their operands transposed from LDS (ds_read_tr).
#include "state_tiles.h"

using namespace vx;

namespace {

constexpr int FEW = 16;        // rows of a sequence up to which it is walked
constexpr int SUB = 64;
constexpr int TS = 8;          // rows staged at a time by step_kernel
constexpr int VB = 128, DB = 64;  // columns of a workgroup's V, of chunk_kernel's K
constexpr int LDV = VB + 8, LDK = DB + 8, LDP = SUB + 8;  // LDS rows (elements)

struct DecayArgs {
    vx_decay_args p;
    const int32_t *cu, *pos, *slots;
    int n_seqs, one_token;
    int max_rows;     // step_kernel: sequences with more rows are left out
    int subs;         // sub-chunks of a chunk
    // [chunks][heads][dim / 32][vdim / 16][64 lanes][8]: what a chunk adds to the state, in the order in which a wave's lanes hold it as
    // an operand (lane: column lane % 16, rows 8 (lane / 16) ..); then, in its place, the state before the chunk as eight high and
    // eight low bfloat16 parts per lane
    float *h;
};

// ---------------------------------------------------------------- few rows
// Thread: columns 4 (tid % 8) .. of the workgroup's 32, state rows tid / 8 + 32 i.
template <typename T, int RD>
__global__ void __launch_bounds__(256) step_kernel(DecayArgs a) {
    extern __shared__ float s_dyn[];  // q [TS][dim] | k [TS][dim] | v [TS][32] | partial outputs [TS][4][32]
    const vx_decay_args &p = a.p;
    const int seq = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 32, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int row0 = a.one_token ? seq : a.cu[seq], len = a.one_token ? 1 : a.cu[seq + 1] - row0;
    if (len > a.max_rows) return;
    const int cols = min(32, p.vdim - c0), c = tid & 7, d0 = tid >> 3;
    const bool live = c * 4 < cols;
    float *sq = s_dyn, *sk = sq + TS * p.dim, *sv = sk + TS * p.dim, *so = sv + TS * 32;
    float *state = p.state + (((size_t)a.slots[seq] * p.heads + h) * p.dim + d0) * p.vdim + c0 + c * 4;
    f32x4 S[RD];
    const bool old = a.pos[row0] > 0;
#pragma unroll
    for (int i = 0; i < RD; i++)
        S[i] = old && live && d0 + i * 32 < p.dim ? *(const f32x4 *)(state + (size_t)i * 32 * p.vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
    const float dm1 = p.decay[2 * h];
    for (int t0 = 0; t0 < len; t0 += TS) {
        const int tn = min(TS, len - t0);
        __syncthreads();
        for (int i = tid; i < tn * p.dim; i += 256) {
            const int t = i / p.dim, d = i - t * p.dim;
            sq[i] = (float)((const T *)p.q)[(size_t)(row0 + t0 + t) * p.ldq + h * p.dim + d];
            sk[i] = (float)((const T *)p.k)[(size_t)(row0 + t0 + t) * p.ldk + h * p.dim + d];
        }
        for (int i = tid; i < tn * 32; i += 256)
            sv[i] = (i & 31) < cols ? (float)((const T *)p.v)[(size_t)(row0 + t0 + (i >> 5)) * p.ldv + h * p.vdim + c0 + (i & 31)] : 0.f;
        __syncthreads();
        for (int t = 0; t < tn; t++) {
            const f32x4 v = *(const f32x4 *)(sv + t * 32 + c * 4);
            f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < RD; i++) {
                const int d = min(d0 + i * 32, p.dim - 1);
                const float k = sk[t * p.dim + d], q = d0 + i * 32 < p.dim ? sq[t * p.dim + d] : 0.f;
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    S[i][e] = fmaf(k, v[e], fmaf(S[i][e], dm1, S[i][e]));
                    o[e] = fmaf(q, S[i][e], o[e]);
                }
            }
#pragma unroll
            for (int e = 0; e < 4; e++) {
                o[e] += __shfl_xor(o[e], 8, 64);
                o[e] += __shfl_xor(o[e], 16, 64);
                o[e] += __shfl_xor(o[e], 32, 64);
            }
            if (lane < 8) *(f32x4 *)(so + (t * 4 + wave) * 32 + lane * 4) = o;
        }
        __syncthreads();
        for (int i = tid; i < tn * 32; i += 256) {
            const int t = i >> 5, x = i & 31;
            if (x < cols) p.out[(size_t)(row0 + t0 + t) * p.ldo + h * p.vdim + c0 + x] = so[(t * 4) * 32 + x] + so[(t * 4 + 1) * 32 + x] + so[(t * 4 + 2) * 32 + x] + so[(t * 4 + 3) * 32 + x];
        }
    }
#pragma unroll
    for (int i = 0; i < RD; i++)
        if (live && d0 + i * 32 < p.dim) *(f32x4 *)(state + (size_t)i * 32 * p.vdim) = S[i];
}

// ---------------------------------------------------------------- many rows
// Rows r0 .. r0 + 63 (zeros from `rows` on) of columns c0 .. c0 + COLS - 1 (zeros from `cols` on) into LDS.
template <int COLS>
__device__ __forceinline__ void stage(bf16 *dst, int ld, const bf16 *src, int ldsrc, int rows, int cols, int tid) {
    constexpr int CP = COLS / 8;
#pragma unroll
    for (int k = 0; k < SUB * CP / 256; k++) {
        const int i = tid + k * 256, r = i / CP, c = i % CP * 8;
        bf16x8 v;
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = (bf16)0.f;
        if (r < rows && c < cols) v = *(const bf16x8 *)(src + (size_t)r * ldsrc + c);
        *(bf16x8 *)(dst + r * ld + c) = v;
    }
}

__global__ void __launch_bounds__(256) chunk_kernel(DecayArgs a) {
    __shared__ bf16 s_k[SUB * LDK], s_v[SUB * LDV];
    const vx_decay_args &p = a.p;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y;
    const int vbs = (p.vdim + VB - 1) / VB, v0 = blockIdx.z % vbs * VB, d0 = blockIdx.z / vbs * DB;
    int seq, ci, chunks;
    if (!item_of_seq(a.cu, a.n_seqs, a.subs * SUB, FEW + 1, blockIdx.x, &seq, &ci, &chunks)) return;
    const int row0 = a.cu[seq] + ci * a.subs * SUB, len = min(a.subs * SUB, a.cu[seq + 1] - row0);
    const float lg = p.decay[2 * h + 1];
    const int tiles = min(VB, p.vdim - v0) / 16;
    f32x4 acc[VB / 16];
#pragma unroll
    for (int v = 0; v < VB / 16; v++) acc[v] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int t0 = 0; t0 < len; t0 += SUB) {
        if (t0) __syncthreads();
        stage<DB>(s_k, LDK, (const bf16 *)p.k + (size_t)(row0 + t0) * p.ldk + h * p.dim + d0, p.ldk, len - t0, p.dim - d0, tid);
        stage<VB>(s_v, LDV, (const bf16 *)p.v + (size_t)(row0 + t0) * p.ldv + h * p.vdim + v0, p.ldv, len - t0, p.vdim - v0, tid);
        __syncthreads();
#pragma unroll
        for (int ks = 0; ks < SUB / 32; ks++) {
            const bf16x8 k = column8(s_k, LDK, ks * 32, wave * 16, lane);
            bf16x8 hi, lo;
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const int t = t0 + ks * 32 + (lane >> 4) * 8 + j;  // (rows beyond the chunk: zeros in LDS, a finite factor)
                bf16 x, y;
                split((float)k[j] * __builtin_amdgcn_exp2f((float)max(len - 1 - t, 0) * lg), &x, &y);
                hi[j] = x, lo[j] = y;
            }
#pragma unroll
            for (int v = 0; v < VB / 16; v++) {
                if (v >= tiles) break;
                const bf16x8 vt = column8(s_v, LDV, ks * 32, v * 16, lane);
                acc[v] = mma(hi, vt, acc[v]);
                acc[v] = mma(lo, vt, acc[v]);
            }
        }
    }
    // rows d0 + 16 wave + 4 (lane / 16) .. of columns lane % 16: four of the eight elements of a lane of the operand
    const int d = d0 + wave * 16 + (lane >> 4) * 4;
    if (d >= p.dim) return;
    float *out = a.h + (size_t)(blockIdx.x * p.heads + h) * p.dim * p.vdim + ((size_t)(d >> 5) * (p.vdim >> 4) + (v0 >> 4)) * 512 +
                 (((d & 31) >> 3) * 16 + (lane & 15)) * 8 + (d & 7);
#pragma unroll
    for (int v = 0; v < VB / 16; v++)
        if (v < tiles) *(f32x4 *)(out + v * 512) = acc[v];
}

// Eight rows of one state column per thread: a lane's part of an operand.
__global__ void __launch_bounds__(256) carry_kernel(DecayArgs a) {
    const vx_decay_args &p = a.p;
    const int seq = blockIdx.x, h = blockIdx.y, per = p.dim * p.vdim, e = blockIdx.z * 256 + threadIdx.x;
    const int size = a.subs * SUB, rows = a.cu[seq + 1] - a.cu[seq], chunks = (rows + size - 1) / size;
    if (rows <= FEW || e >= per / 8) return;
    int first = 0;
    for (int s = 0; s < seq; s++) {
        const int n = a.cu[s + 1] - a.cu[s];
        if (n > FEW) first += (n + size - 1) / size;
    }
    const int lane = e & 63, tile = e >> 6, vt = p.vdim >> 4, d = tile / vt * 32 + (lane >> 4) * 8, v = tile % vt * 16 + (lane & 15);
    float *state = p.state + ((size_t)a.slots[seq] * p.heads + h) * per + (size_t)d * p.vdim + v;
    float *hp = a.h + (size_t)(first * p.heads + h) * per + (size_t)e * 8;
    const size_t step = (size_t)p.heads * per;
    const bool old = a.pos[a.cu[seq]] > 0;
    float S[8];
#pragma unroll
    for (int j = 0; j < 8; j++) S[j] = old ? state[(size_t)j * p.vdim] : 0.f;
    const float lg = p.decay[2 * h + 1], whole = __builtin_amdgcn_exp2f((float)size * lg);
    constexpr int U = 4;
    for (int k = 0; k < chunks; k += U) {
        f32x4 own[U][2];
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int x = 0; x < 2; x++) own[u][x] = *(const f32x4 *)(hp + (size_t)min(k + u, chunks - 1) * step + x * 4);
#pragma unroll
        for (int u = 0; u < U; u++) {
            if (k + u >= chunks) break;
            bf16x8 hi, lo;
#pragma unroll
            for (int j = 0; j < 8; j++) {
                bf16 x, y;
                split(S[j], &x, &y);
                hi[j] = x, lo[j] = y;
            }
            bf16x8 *at = (bf16x8 *)(hp + (size_t)(k + u) * step);
            at[0] = hi, at[1] = lo;
            const float f = k + u + 1 < chunks ? whole : __builtin_amdgcn_exp2f((float)(rows - (chunks - 1) * size) * lg);
#pragma unroll
            for (int j = 0; j < 8; j++) S[j] = fmaf(f, S[j], own[u][j >> 2][j & 3]);
        }
    }
#pragma unroll
    for (int j = 0; j < 8; j++) state[(size_t)j * p.vdim] = S[j];
}

__global__ void __launch_bounds__(256) out_kernel(DecayArgs a) {
    __shared__ bf16 s_v[SUB * LDV], s_hi[SUB * LDP], s_lo[SUB * LDP];
    const vx_decay_args &p = a.p;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y, v0 = blockIdx.z * VB;
    const int q4 = (lane >> 4) * 4, q8 = (lane >> 4) * 8, l16 = lane & 15;
    int id = blockIdx.x, seq = 0, first = 0;  // sub-chunks of the sequences one after the other; first: chunks before the sequence
    for (;; seq++) {
        if (seq >= a.n_seqs) return;
        const int n = a.cu[seq + 1] - a.cu[seq];
        if (n <= FEW) continue;
        const int subs = (n + SUB - 1) / SUB;
        if (id < subs) break;
        id -= subs, first += (subs + a.subs - 1) / a.subs;
    }
    const int chunk = id / a.subs, b = id % a.subs;
    const int row0 = a.cu[seq] + chunk * a.subs * SUB, len = min(a.subs * SUB, a.cu[seq + 1] - row0);  // the chunk
    const int i0 = b * SUB, n_rows = min(SUB, len - i0);                                               // the sub-chunk in it
    const float lg = p.decay[2 * h + 1];
    const bf16 *q = (const bf16 *)p.q + (size_t)row0 * p.ldq + h * p.dim + q8, *k = (const bf16 *)p.k + (size_t)row0 * p.ldk + h * p.dim + q8;
    const int tiles = min(VB, p.vdim - v0) / 16;
    f32x4 acc[2][4];  // columns v0 + 16 (2 wave + x) + q4 .. of rows 16 it + l16
#pragma unroll
    for (int x = 0; x < 2; x++)
#pragma unroll
        for (int it = 0; it < 4; it++) acc[x][it] = f32x4{0.f, 0.f, 0.f, 0.f};
    if ((chunk > 0 || a.pos[row0] > 0) && wave * 2 < tiles) {  // (a chunk behind the first starts at a position above 0 as well)
        const bf16x8 *S = (const bf16x8 *)(a.h + (size_t)((first + chunk) * p.heads + h) * p.dim * p.vdim) + lane * 2;
        int tile[2];
#pragma unroll
        for (int x = 0; x < 2; x++) tile[x] = (v0 >> 4) + min(wave * 2 + x, tiles - 1);
        bf16x8 hi[2], lo[2], qf[4];
        const auto fetch = [&](int ds) {
#pragma unroll
            for (int x = 0; x < 2; x++) {
                const bf16x8 *at = S + ((size_t)(ds >> 5) * (p.vdim >> 4) + tile[x]) * 128;
                hi[x] = at[0], lo[x] = at[1];
            }
#pragma unroll
            for (int it = 0; it < 4; it++) qf[it] = *(const bf16x8 *)(q + (size_t)min(i0 + it * 16 + l16, len - 1) * p.ldq + ds);
        };
        fetch(0);
        for (int ds = 0; ds < p.dim; ds += 32) {
            bf16x8 ch[2], cl[2], cq[4];
#pragma unroll
            for (int x = 0; x < 2; x++) ch[x] = hi[x], cl[x] = lo[x];
#pragma unroll
            for (int it = 0; it < 4; it++) cq[it] = qf[it];
            if (ds + 32 < p.dim) fetch(ds + 32);
#pragma unroll
            for (int x = 0; x < 2; x++)
#pragma unroll
                for (int it = 0; it < 4; it++) {
                    acc[x][it] = mma(ch[x], cq[it], acc[x][it]);
                    acc[x][it] = mma(cl[x], cq[it], acc[x][it]);
                }
        }
#pragma unroll
        for (int it = 0; it < 4; it++) {
            const float f = __builtin_amdgcn_exp2f((float)(i0 + it * 16 + l16 + 1) * lg);
#pragma unroll
            for (int x = 0; x < 2; x++) acc[x][it] *= f;
        }
    }
    const int own = min(i0 + wave * 16 + l16, len - 1);  // this wave's row whose scores it computes, in the chunk
    for (int kb = 0; kb <= b; kb++) {
        if (kb) __syncthreads();
        stage<VB>(s_v, LDV, (const bf16 *)p.v + (size_t)(row0 + kb * SUB) * p.ldv + h * p.vdim + v0, p.ldv, len - kb * SUB, p.vdim - v0, tid);
#pragma unroll
        for (int g = 0; g < 2; g++) {
            if (kb == b && g * 32 > wave * 16 + 15) break;
            // keys 32 g + 8 (i / 4) + 4 t + i % 4 for lane i of tile t: a lane ends with eight neighbouring keys of one row
            const int key = kb * SUB + g * 32 + (l16 >> 2) * 8 + (l16 & 3);
            const bf16 *kp[2] = {k + (size_t)min(key, len - 1) * p.ldk, k + (size_t)min(key + 4, len - 1) * p.ldk};
            f32x4 st[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
            const bf16 *qp = q + (size_t)own * p.ldq;
            for (int ds = 0; ds < p.dim; ds += 32) {
                const bf16x8 qf = *(const bf16x8 *)(qp + ds);
                st[0] = mma(*(const bf16x8 *)(kp[0] + ds), qf, st[0]);
                st[1] = mma(*(const bf16x8 *)(kp[1] + ds), qf, st[1]);
            }
            const int j0 = kb * SUB + g * 32 + q8, i = i0 + wave * 16 + l16;
            bf16x8 hi, lo;
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const int back = i - (j0 + j);
                const float s = back >= 0 ? (j < 4 ? st[0][j & 3] : st[1][j & 3]) * __builtin_amdgcn_exp2f((float)back * lg) : 0.f;
                bf16 y, z;
                split(s, &y, &z);
                hi[j] = y, lo[j] = z;
            }
            *(bf16x8 *)(s_hi + (wave * 16 + l16) * LDP + g * 32 + q8) = hi;
            *(bf16x8 *)(s_lo + (wave * 16 + l16) * LDP + g * 32 + q8) = lo;
        }
        __syncthreads();
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            bf16x8 vt[2];
#pragma unroll
            for (int x = 0; x < 2; x++) vt[x] = column8(s_v, LDV, ks * 32, min(wave * 2 + x, tiles - 1) * 16, lane);
#pragma unroll
            for (int it = 0; it < 4; it++) {
                if (kb == b && ks * 32 > it * 16 + 15) continue;
                const bf16x8 hi = *(const bf16x8 *)(s_hi + (it * 16 + l16) * LDP + ks * 32 + q8);
                const bf16x8 lo = *(const bf16x8 *)(s_lo + (it * 16 + l16) * LDP + ks * 32 + q8);
#pragma unroll
                for (int x = 0; x < 2; x++) {
                    acc[x][it] = mma(vt[x], hi, acc[x][it]);
                    acc[x][it] = mma(vt[x], lo, acc[x][it]);
                }
            }
        }
    }
#pragma unroll
    for (int it = 0; it < 4; it++) {
        if (it * 16 + l16 >= n_rows) continue;
        float *out = p.out + (size_t)(row0 + i0 + it * 16 + l16) * p.ldo + h * p.vdim + v0 + q4;
#pragma unroll
        for (int x = 0; x < 2; x++)
            if (wave * 2 + x < tiles) *(f32x4 *)(out + (wave * 2 + x) * 16) = acc[x][it];
    }
}

template <typename T>
void launch_step(vx_backend *be, const DecayArgs &a) {
    const dim3 grid(a.n_seqs, a.p.heads, ceil_div(a.p.vdim, 32));
    const size_t lds = (size_t)TS * (2 * a.p.dim + 5 * 32) * 4;
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

// ---------------------------------------------------------------- norm with a gate
// A row per workgroup; NV > 0: cols is a multiple of 4 and at most 4 * NV * blockDim.x, everything aligned: a row lives in registers.
template <typename T, int NV>
__global__ void __launch_bounds__(1024) gated_norm_kernel(const float *x, int ldx, const float *gate, int ldg, const float *w, float eps, int cols,
                                                          int count, T *out, int ldo) {
    __shared__ float sm[16];
    const int tid = threadIdx.x, nt = blockDim.x;
    x += (size_t)blockIdx.x * ldx, gate += (size_t)blockIdx.x * ldg, out += (size_t)blockIdx.x * ldo;
    const auto inverse = [&](float ss) {
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
        if ((tid & 63) == 0) sm[tid >> 6] = ss;
        __syncthreads();
        float t = 0.f;
        for (int i = 0; i < (nt >> 6); i++) t += sm[i];
        return 1.0f / sqrtf(t / (float)count + eps);
    };
    float ss = 0.f;
    if constexpr (NV > 0) {
        f32x4 v[NV], g[NV];
        const int n4 = cols >> 2;
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = tid + i * nt;
            v[i] = c < n4 ? ((const f32x4 *)x)[c] : f32x4{0.f, 0.f, 0.f, 0.f};
            if (c < n4) g[i] = ((const f32x4 *)gate)[c];
#pragma unroll
            for (int e = 0; e < 4; e++) ss = fmaf(v[i][e], v[i][e], ss);
        }
        const float inv = inverse(ss);
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = tid + i * nt;
            if (c < n4) {
                f32x4 o = v[i] * inv * ((const f32x4 *)w)[c];
#pragma unroll
                for (int e = 0; e < 4; e++) o[e] *= sigmoid_f(g[i][e]);
                store4(out + c * 4, o);
            }
        }
    } else {
        for (int c = tid; c < cols; c += nt) ss = fmaf(x[c], x[c], ss);
        const float inv = inverse(ss);
        for (int c = tid; c < cols; c += nt) out[c] = (T)(x[c] * inv * w[c] * sigmoid_f(gate[c]));
    }
    for (int c = cols + tid; c < ldo; c += nt) out[c] = (T)0.f;
}

template <typename T>
void launch_gated(vx_backend *be, const float *x, int ldx, const float *gate, int ldg, const float *w, float eps, int rows, int cols, int count, T *out,
                  int ldo) {
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = cols % 4 == 0 && ldx % 4 == 0 && ldg % 4 == 0 && ldo % 4 == 0 && al(x) && al(gate) && al(w) && al(out);
    const int n4 = cols / 4;
    int threads = rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads / 2 >= n4) threads /= 2;
    while (threads < 1024 && n4 > 4 * threads) threads *= 2;
    const int nv = ceil_div(n4, threads);
    if (!vec || nv > 4)
        gated_norm_kernel<T, 0><<<rows, 1024, 0, be->stream>>>(x, ldx, gate, ldg, w, eps, cols, count, out, ldo);
    else if (nv <= 1)
        gated_norm_kernel<T, 1><<<rows, threads, 0, be->stream>>>(x, ldx, gate, ldg, w, eps, cols, count, out, ldo);
    else if (nv <= 2)
        gated_norm_kernel<T, 2><<<rows, threads, 0, be->stream>>>(x, ldx, gate, ldg, w, eps, cols, count, out, ldo);
    else
        gated_norm_kernel<T, 4><<<rows, threads, 0, be->stream>>>(x, ldx, gate, ldg, w, eps, cols, count, out, ldo);
}

}  // namespace

extern "C" {

int vx_decay_attn(vx_backend *be, int act, const vx_ragged *b, const vx_decay_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_decay_attn");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_decay_attn: unknown activation type %d", act);
    VX_REQUIRE(p && p->heads >= 1 && p->heads <= 65535 && p->dim >= 32 && p->dim % 32 == 0 && p->dim <= 512 && p->vdim >= 16 && p->vdim % 16 == 0 &&
                   p->vdim <= 512,
               "vx_decay_attn: bad heads");
    VX_REQUIRE(p->decay && p->q && p->k && p->v && p->state && p->out, "vx_decay_attn: null argument");
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    VX_REQUIRE(p->ldq >= p->heads * p->dim && p->ldk >= p->heads * p->dim && p->ldv >= p->heads * p->vdim && p->ldo >= p->heads * p->vdim &&
                   p->ldq % 8 == 0 && p->ldk % 8 == 0 && p->ldv % 8 == 0 && p->ldo % 4 == 0 && al(p->q) && al(p->k) && al(p->v) && al(p->state) && al(p->out),
               "vx_decay_attn: bad strides or alignment");
    DecayArgs a{*p, b->cu_seqlens, b->token_pos, b->table_rows, b->n_seqs, b->q_lens ? 0 : 1, FEW, 1, nullptr};
    bool few = !b->q_lens, many = false;
    int64_t rows = 0;
    if (b->q_lens)
        for (int s = 0; s < b->n_seqs; s++) {
            if (b->q_lens[s] <= FEW)
                few = true;
            else
                many = true, rows += b->q_lens[s];
        }
    if (act == VX_ACT_F32) few = true, many = false, a.max_rows = 1 << 30;
    if (many) {
        // two sub-chunks to a chunk halve the states that pass through memory, where enough workgroups are left
        a.subs = rows / SUB * p->heads >= 1024 ? 2 : 1;
        const int chunks = count_items(b, a.subs * SUB, FEW + 1), subs = count_items(b, SUB, FEW + 1);
        rc = ensure_ws(be, &be->scan_ws, &be->scan_ws_bytes, (size_t)chunks * p->heads * p->dim * p->vdim * 4, "scan");
        if (rc) return rc;
        a.h = (float *)be->scan_ws;
        chunk_kernel<<<dim3(chunks, p->heads, ceil_div(p->vdim, VB) * ceil_div(p->dim, DB)), 256, 0, be->stream>>>(a);
        VX_CHECK_LAUNCH();
        carry_kernel<<<dim3(b->n_seqs, p->heads, ceil_div(p->dim * p->vdim, 2048)), 256, 0, be->stream>>>(a);
        VX_CHECK_LAUNCH();
        out_kernel<<<dim3(subs, p->heads, ceil_div(p->vdim, VB)), 256, 0, be->stream>>>(a);
        VX_CHECK_LAUNCH();
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

int vx_gated_norm(vx_backend *be, int act, const float *x, int ldx, const float *gate, int ldg, const float *w, float eps, int rows, int cols,
                  int count, void *out, int ldo) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_gated_norm: unknown activation type %d", act);
    VX_REQUIRE(x && gate && w && out && rows >= 1 && cols >= 1 && count >= 1 && count <= cols && ldx >= cols && ldg >= cols && ldo >= cols,
               "vx_gated_norm: bad arguments");
    if (act == VX_ACT_BF16)
        launch_gated<bf16>(be, x, ldx, gate, ldg, w, eps, rows, cols, count, (bf16 *)out, ldo);
    else
        launch_gated<float>(be, x, ldx, gate, ldg, w, eps, rows, cols, count, (float *)out, ldo);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
