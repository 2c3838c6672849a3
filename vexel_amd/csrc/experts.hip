// Routing of mixtures of experts (vx_route): which experts a row takes, and the (row, choice) pairs in the experts' order. The
// experts' maps themselves are linear.hip's.
//
//  * choose: a wave per row. Every lane ranks its experts among all by counting, so that nothing waits for a chain of maxima.
//  * place: one workgroup counts, adds up and deals out places; its atomics are in LDS. The order of an expert's rows among
//    themselves does not matter to anyone's result.
// Few rows (a decode step): one workgroup does both, and the choices stay in LDS between them.
#include <type_traits>

#include "ragged.h"

using namespace vx;

namespace {

constexpr int MAX_EXPERTS = 1024;
constexpr int FEW = 64;            // rows that one workgroup chooses for
constexpr int FEW_LDS = 48 * 1024; // bytes it may keep them in
constexpr int THREADS = 1024;

__device__ __forceinline__ float score(const vx_route_args &p, int row, int e) {
    const float *z = p.z + (size_t)row * p.ldz + e;
    float t = z[0];
#pragma unroll 4
    for (int k = 1; k < p.z_slices; k++) t += z[(size_t)k * p.z_stride];
    if (p.bias) t += p.bias[e];
    return p.softmax ? t : 1.0f / (1.0f + expf(-t));
}

// How many of a[0 .. n - 1] come before element i, which is v: the larger ones, and with TIES equal ones of a lower index. Reads up to
// three elements beyond n - 1, which have to be -infinity.
template <bool TIES>
__device__ __forceinline__ int rank_of(const float *a, int n, float v, int i) {
    int rank = 0;
#pragma unroll 4
    for (int k = 0; k < n; k += 4) {
        const f32x4 x = *(const f32x4 *)(a + k);
#pragma unroll
        for (int e = 0; e < 4; e++) rank += x[e] > v || (TIES && x[e] == v && k + e < i);
    }
    return rank;
}

__host__ __device__ __forceinline__ int up4(int n) { return (n + 3) & ~3; }

// c: [up4(experts)] choice scores of the row in LDS, s: its scores, g: [up4(groups)]; this wave's own. chosen, weights: [top].
__device__ __forceinline__ void choose_row(const vx_route_args &p, int lane, float *c, const float *s, float *g, int32_t *chosen, float *weights) {
    if (p.groups > 1) {
        const int size = p.experts / p.groups;
        for (int i = lane; i < up4(p.groups); i += 64) {
            float a = -INFINITY, b = -INFINITY;
            if (i < p.groups)
#pragma unroll 4
                for (int k = 0; k < size; k++) {
                    const float v = c[i * size + k];
                    b = fmaxf(b, fminf(a, v));
                    a = fmaxf(a, v);
                }
            g[i] = size > 1 ? a + b : a;
        }
        __builtin_amdgcn_wave_barrier();
        for (int e = lane; e < p.experts; e += 64) {
            const int own = e / size;
            if (rank_of<true>(g, p.groups, g[own], own) >= p.keep) c[e] = -INFINITY;
        }
        __builtin_amdgcn_wave_barrier();
    }
    // The experts that fewer than `top` others surpass, in the order of their numbers; more than `top` when the last of them has an
    // equal: then equals rank by number.
    // Softmax: relative to the largest s of all (with no correction that is the first choice), and divided by their sum in a second round.
    float top_s = -INFINITY, inv = 1.0f;
    if (p.softmax) {
        for (int e = lane; e < p.experts; e += 64) top_s = fmaxf(top_s, s[e]);
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) top_s = fmaxf(top_s, __shfl_xor(top_s, off, 64));
    }
    const auto weight = [&](int e) { return p.softmax ? expf(s[e] - top_s) : s[e]; };
    float sum = 0.f;  // of this lane's
    const auto deal = [&](auto ties) {
        int n = 0;
        sum = 0.f;
        for (int e0 = 0; e0 < p.experts; e0 += 64) {
            const int e = e0 + lane;
            const bool takes = e < p.experts && rank_of<decltype(ties)::value>(c, p.experts, c[min(e, p.experts - 1)], e) < p.top;
            const uint64_t mask = __ballot(takes);
            const int slot = n + __popcll(mask & (((uint64_t)1 << lane) - 1));
            if (takes && slot < p.top) {
                const float w = weight(e);
                chosen[slot] = e, weights[slot] = w * inv, sum += w;
            }
            n += __popcll(mask);
        }
        return n;
    };
    const bool ties = deal(std::false_type()) != p.top;
    if (ties) deal(std::true_type());
    if (p.softmax) {
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
        inv = 1.0f / sum;
        if (ties)
            deal(std::true_type());
        else
            deal(std::false_type());
    }
    __builtin_amdgcn_wave_barrier();
}

// chosen [rows][top] -> places, order, tiles. chosen may be p.places itself (every pair is read before its place is written). One
// workgroup of THREADS threads.
__device__ __forceinline__ void place_rows(const vx_route_args &p, const int32_t *chosen, int *count, int *first, int *scan) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, pairs = p.rows * p.top;
    for (int e = tid; e < MAX_EXPERTS; e += THREADS) count[e] = 0;
    __syncthreads();
    for (int i = tid; i < pairs; i += THREADS) atomicAdd(&count[chosen[i]], 1);
    __syncthreads();
    // two prefix sums over the experts at once: places, tiles
    const int n = tid < p.experts ? count[tid] : 0, t = (n + p.tile_rows - 1) / p.tile_rows;
    int a = n, b = t;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const int x = __shfl_up(a, off, 64), y = __shfl_up(b, off, 64);
        if (lane >= off) a += x, b += y;
    }
    if (lane == 63) scan[wave] = a, scan[16 + wave] = b;
    __syncthreads();
    int pa = 0, pb = 0, tiles = 0;
    for (int w = 0; w < 16; w++) {
        if (w < wave) pa += scan[w], pb += scan[16 + w];
        tiles += scan[16 + w];
    }
    const int at = pa + a - n, tile = pb + b - t;
    if (tid < p.experts) {
        first[tid] = at;
        for (int k = 0; k < t; k++) {
            int32_t *r = p.tiles + 4 + 4 * (tile + k);
            r[0] = tid, r[1] = at + k * p.tile_rows, r[2] = min(p.tile_rows, n - k * p.tile_rows), r[3] = 0;
        }
    }
    const int more = p.shared ? (p.rows + p.tile_rows - 1) / p.tile_rows : 0;
    for (int k = tid; k < more; k += THREADS) {
        int32_t *r = p.tiles + 4 + 4 * (tiles + k);
        r[0] = p.experts, r[1] = pairs + k * p.tile_rows, r[2] = min(p.tile_rows, p.rows - k * p.tile_rows), r[3] = 0;
    }
    if (tid == 0) p.tiles[0] = tiles + more;
    __syncthreads();
    for (int i = tid; i < pairs; i += THREADS) {
        const int place = atomicAdd(&first[chosen[i]], 1);
        p.order[place] = i / p.top;
        p.places[i] = place;
    }
    if (p.shared)
        for (int i = tid; i < p.rows; i += THREADS) p.order[pairs + i] = i;
}

// dynamic LDS: per wave choice scores | scores | groups' sums
__global__ void __launch_bounds__(256) route_choose_kernel(vx_route_args p) {
    extern __shared__ float s_dyn[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row = blockIdx.x * 4 + wave, ne = up4(p.experts);
    float *c = s_dyn + (size_t)wave * (2 * ne + up4(p.groups)), *s = c + ne;
    if (row >= p.rows) return;  // (nothing is shared between waves)
    for (int e = lane; e < ne; e += 64) {
        const float t = e < p.experts ? score(p, row, e) : 0.f;
        s[e] = t;
        c[e] = e < p.experts ? (p.correction ? t + p.correction[e] : t) : -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
    choose_row(p, lane, c, s, s + ne, p.places + (size_t)row * p.top, p.weights + (size_t)row * p.top);
}

__global__ void __launch_bounds__(THREADS) route_place_kernel(vx_route_args p) {
    __shared__ int count[MAX_EXPERTS], first[MAX_EXPERTS], scan[32];
    place_rows(p, p.places, count, first, scan);
}

// dynamic LDS: [rows] choice scores | [rows] scores | per wave groups' sums | [rows][top] choices
__global__ void __launch_bounds__(THREADS) route_few_kernel(vx_route_args p) {
    extern __shared__ float s_dyn[];
    __shared__ int count[MAX_EXPERTS], first[MAX_EXPERTS], scan[32];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, ne = up4(p.experts);
    float *c = s_dyn, *s = c + p.rows * ne, *g = s + p.rows * ne;
    int32_t *chosen = (int32_t *)(g + THREADS / 64 * up4(p.groups));
    for (int i = threadIdx.x; i < p.rows * ne; i += THREADS) {
        const int row = i / ne, e = i - row * ne;
        const float t = e < p.experts ? score(p, row, e) : 0.f;
        s[i] = t;
        c[i] = e < p.experts ? (p.correction ? t + p.correction[e] : t) : -INFINITY;
    }
    __syncthreads();
    for (int row = wave; row < p.rows; row += THREADS / 64)
        choose_row(p, lane, c + row * ne, s + row * ne, g + wave * up4(p.groups), chosen + row * p.top, p.weights + (size_t)row * p.top);
    __syncthreads();
    place_rows(p, chosen, count, first, scan);
}

}  // namespace

extern "C" {

int vx_route_max_tiles(int rows, int experts, int top, int shared, int tile_rows) {
    if (rows < 1 || experts < 1 || top < 1 || tile_rows < 1) return 0;
    const int64_t pairs = (int64_t)rows * top;
    return (int)((pairs < experts ? pairs : experts) + pairs / tile_rows + (shared ? ceil_div(rows, tile_rows) : 0));
}

int vx_route(vx_backend *be, const vx_route_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(p && p->rows >= 1 && p->z && p->z_slices >= 1 && p->weights && p->places && p->order && p->tiles && p->tile_rows >= 1,
               "vx_route: bad arguments");
    VX_REQUIRE(p->experts >= 1 && p->experts <= MAX_EXPERTS && p->ldz >= p->experts, "vx_route: %d experts (at most %d)", p->experts, MAX_EXPERTS);
    vx_route_args a = *p;
    if (a.groups < 1) a.groups = 1;
    VX_REQUIRE(a.experts % a.groups == 0 && (a.groups == 1 || (a.keep >= 1 && a.keep <= a.groups)), "vx_route: %d of %d groups of %d experts", a.keep, a.groups,
               a.experts);
    VX_REQUIRE(a.top >= 1 && a.top <= (a.groups == 1 ? a.experts : a.keep * (a.experts / a.groups)), "vx_route: %d of %d experts", a.top, a.experts);
    VX_REQUIRE((int64_t)a.rows * (a.top + 1) < ((int64_t)1 << 30), "vx_route: %d rows", a.rows);
    const size_t few = ((size_t)a.rows * (2 * up4(a.experts) + a.top) + THREADS / 64 * up4(a.groups)) * 4;
    if (a.rows <= FEW && few <= FEW_LDS) {
        route_few_kernel<<<1, THREADS, few, be->stream>>>(a);
    } else {
        route_choose_kernel<<<ceil_div(a.rows, 4), 256, 4 * (size_t)(2 * up4(a.experts) + up4(a.groups)) * 4, be->stream>>>(a);
        VX_CHECK_LAUNCH();
        route_place_kernel<<<1, THREADS, 0, be->stream>>>(a);
    }
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
