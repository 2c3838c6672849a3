// The pieces of mixed-batch layers beside linear maps and attention: the norm | residual | norm seam (which also adds experts'
// rows), the residual | norm | average over the depth seam, the normed polynomial activation, the causal depthwise convolution and the selective scan. All of them in float32 on activations that are bfloat16 or float32 (T).
//
// Scan: a lane keeps 8 states of one channel in registers, LP = padded / 8 neighbouring lanes make up the channel. A
// sequence's rows are cut into chunks of CHUNK; where a sequence has several, a first pass finds what every chunk adds to
// the state on its own, a second one runs over the chunks, and the last computes the outputs from the states before them.
// A chunk's end depends on its length in the sequence only through rounding.
#include "ragged.h"

using namespace vx;

namespace {

__device__ __forceinline__ float block_sum(float v, float *sm) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    __syncthreads();  // (an earlier use of sm is over)
    if ((threadIdx.x & 63) == 0) sm[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < (int)(blockDim.x >> 6); i++) t += sm[i];
    return t;
}

// What row r's experts add to columns c ..: W is a vector of float32 columns.
template <typename T, typename W>
__device__ __forceinline__ void add_experts(const vx_residual_norm_args &p, int r, int c, W *x) {
    const T *rows = (const T *)p.e_rows + c;
    const auto read = [&](size_t place) {
        if constexpr (sizeof(W) == 4) {
            return (W)rows[place * p.lde];
        } else {
            return __builtin_convertvector(*(const typename Vec4<T>::type *)(rows + place * p.lde), f32x4);
        }
    };
    for (int j = 0; j < p.e_top; j++) *x += p.e_weights[(size_t)r * p.e_top + j] * read(p.e_places[(size_t)r * p.e_top + j]);
    if (p.e_shared >= 0) *x += read((size_t)p.e_shared + r);
}

// NV > 0: cols is a multiple of 4 and at most 4 * NV * blockDim.x, everything aligned: a row lives in registers.
template <typename T, int NV>
__global__ void __launch_bounds__(1024) residual_norm_kernel(vx_residual_norm_args p) {
    __shared__ float sm[16];
    const int i = blockIdx.x, r = p.row_idx ? p.row_idx[i] : i, tid = threadIdx.x, nt = blockDim.x;
    const float *xr = p.x_in + (size_t)r * p.cols;
    const float *ar = p.add ? p.add + (size_t)r * p.cols : nullptr;
    float *xo = p.x_out ? p.x_out + (size_t)r * p.cols : nullptr;
    T *out = p.w_pre ? (T *)p.out + (size_t)i * p.ldo : nullptr;
    if constexpr (NV > 0) {
        f32x4 x[NV], y[NV];
        const int n4 = p.cols >> 2;
#pragma unroll
        for (int v = 0; v < NV; v++) {
            const int c = tid + v * nt;
            x[v] = c < n4 ? ((const f32x4 *)xr)[c] : f32x4{0.f, 0.f, 0.f, 0.f};
        }
        if (p.y) {
            float ss = 0.f;
#pragma unroll
            for (int v = 0; v < NV; v++) {
                const int c = tid + v * nt;
                y[v] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (c < n4) {
                    const float *yr = p.y + (size_t)r * p.ldy + c * 4;
                    y[v] = *(const f32x4 *)yr;
                    for (int s = 1; s < p.y_slices; s++) y[v] += *(const f32x4 *)(yr + (size_t)s * p.y_stride);
                }
#pragma unroll
                for (int e = 0; e < 4; e++) ss = fmaf(y[v][e], y[v][e], ss);
            }
            if (p.w_post) {
                const float inv = 1.0f / sqrtf(block_sum(ss, sm) / (float)p.cols + p.eps);
#pragma unroll
                for (int v = 0; v < NV; v++) {
                    const int c = tid + v * nt;
                    if (c < n4) {
                        const f32x4 w = ((const f32x4 *)p.w_post)[c];
#pragma unroll
                        for (int e = 0; e < 4; e++) x[v][e] = fmaf(p.mult, y[v][e] * inv * w[e], x[v][e]);
                    }
                }
            } else {
#pragma unroll
                for (int v = 0; v < NV; v++) {
                    const int c = tid + v * nt;
                    if (c < n4 && p.y_bias) y[v] += ((const f32x4 *)p.y_bias)[c];
#pragma unroll
                    for (int e = 0; e < 4; e++) x[v][e] = fmaf(p.mult, y[v][e], x[v][e]);
                }
            }
        }
        if (p.e_rows)
#pragma unroll
            for (int v = 0; v < NV; v++)
                if (tid + v * nt < n4) add_experts<T>(p, r, (tid + v * nt) * 4, &x[v]);
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < NV; v++) {
            const int c = tid + v * nt;
            if (c < n4) {
                if (ar) x[v] += ((const f32x4 *)ar)[c];
                if (xo) ((f32x4 *)xo)[c] = x[v];
            }
#pragma unroll
            for (int e = 0; e < 4; e++) ss = fmaf(x[v][e], x[v][e], ss);
        }
        if (!out) return;
        const float inv = 1.0f / sqrtf(block_sum(ss, sm) / (float)p.cols + p.eps);
#pragma unroll
        for (int v = 0; v < NV; v++) {
            const int c = tid + v * nt;
            if (c < n4) {
                const f32x4 w = ((const f32x4 *)p.w_pre)[c];
                f32x4 o;
#pragma unroll
                for (int e = 0; e < 4; e++) o[e] = x[v][e] * inv * w[e];
                store4(out + c * 4, o);
            }
        }
    } else {
        // any width: the row is read again for every pass
        auto yat = [&](int c) {
            float t = p.y[(size_t)r * p.ldy + c];
            for (int s = 1; s < p.y_slices; s++) t += p.y[(size_t)s * p.y_stride + (size_t)r * p.ldy + c];
            return t;
        };
        float inv_y = 0.f;
        if (p.y && p.w_post) {
            float ss = 0.f;
            for (int c = tid; c < p.cols; c += nt) {
                const float t = yat(c);
                ss = fmaf(t, t, ss);
            }
            inv_y = 1.0f / sqrtf(block_sum(ss, sm) / (float)p.cols + p.eps);
        }
        auto xat = [&](int c) {
            float t = xr[c];
            if (p.y) t = fmaf(p.mult, p.w_post ? yat(c) * inv_y * p.w_post[c] : p.y_bias ? yat(c) + p.y_bias[c] : yat(c), t);
            if (p.e_rows) add_experts<T>(p, r, c, &t);
            return ar ? t + ar[c] : t;
        };
        float ss = 0.f;
        if (out)
            for (int c = tid; c < p.cols; c += nt) {
                const float t = xat(c);
                ss = fmaf(t, t, ss);
            }
        const float inv = out ? 1.0f / sqrtf(block_sum(ss, sm) / (float)p.cols + p.eps) : 0.f;
        for (int c = tid; c < p.cols; c += nt) {  // (a thread reads and writes its own columns only: x_out may be x_in)
            const float t = xat(c);
            if (xo) xo[c] = t;
            if (out) out[c] = (T)(t * inv * p.w_pre[c]);
        }
    }
    if (out)
        for (int c = p.cols + tid; c < p.ldo; c += nt) out[c] = (T)0.f;
}

// NV as above. The earlier results of a row are read only where it is averaged.
template <typename T, int NV>
__global__ void __launch_bounds__(1024) post_norm_kernel(vx_post_norm_args p) {
    __shared__ float sm[16];
    const int i = blockIdx.x, r = p.row_idx ? p.row_idx[i] : i, tid = threadIdx.x, nt = blockDim.x;
    const float *xr = p.x_in + (size_t)r * p.cols;
    float *xo = p.x_out ? p.x_out + (size_t)r * p.cols : nullptr;
    float *hr = p.n_avg > 0 ? p.hist + (size_t)r * p.cols : nullptr;
    T *out = p.out ? (T *)p.out + (size_t)i * p.ldo : nullptr;
    const float n = (float)p.cols;
    if constexpr (NV > 0) {
        f32x4 x[NV];
        const int n4 = p.cols >> 2;
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < NV; v++) {
            const int c = tid + v * nt;
            x[v] = c < n4 ? ((const f32x4 *)xr)[c] : f32x4{0.f, 0.f, 0.f, 0.f};
            if (p.w && c < n4) {
                const float *yr = p.y + (size_t)r * p.ldy + c * 4;
                f32x4 y = *(const f32x4 *)yr;
                for (int s = 1; s < p.y_slices; s++) y += *(const f32x4 *)(yr + (size_t)s * p.y_stride);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    x[v][e] = fmaf(p.alpha, x[v][e], y[e]);
                    ss = fmaf(x[v][e], x[v][e], ss);
                }
            }
        }
        if (p.w) {
            const float inv = 1.0f / sqrtf(block_sum(ss, sm) / n + p.eps);
#pragma unroll
            for (int v = 0; v < NV; v++) {
                const int c = tid + v * nt;
                if (c < n4) x[v] = x[v] * inv * ((const f32x4 *)p.w)[c];
            }
        }
        if (hr) {
            if (p.keep)
#pragma unroll
                for (int v = 0; v < NV; v++) {
                    const int c = tid + v * nt;
                    if (c < n4) ((f32x4 *)(hr + (size_t)(p.n_avg - 1) * p.hist_stride))[c] = x[v];
                }
            const float own = p.avg[p.n_avg - 1];
#pragma unroll
            for (int v = 0; v < NV; v++) x[v] *= own;
            for (int j = 0; j + 1 < p.n_avg; j++) {
                const float w = p.avg[j];
#pragma unroll
                for (int v = 0; v < NV; v++) {
                    const int c = tid + v * nt;
                    if (c < n4) x[v] += w * ((const f32x4 *)(hr + (size_t)j * p.hist_stride))[c];
                }
            }
        }
        if (xo)
#pragma unroll
            for (int v = 0; v < NV; v++) {
                const int c = tid + v * nt;
                if (c < n4) ((f32x4 *)xo)[c] = x[v];
            }
        if (!out) return;
        float inv = 1.0f;
        if (p.w_pre) {
            ss = 0.f;
#pragma unroll
            for (int v = 0; v < NV; v++)
#pragma unroll
                for (int e = 0; e < 4; e++) ss = fmaf(x[v][e], x[v][e], ss);
            inv = 1.0f / sqrtf(block_sum(ss, sm) / n + p.eps);
        }
#pragma unroll
        for (int v = 0; v < NV; v++) {
            const int c = tid + v * nt;
            if (c < n4) store4(out + c * 4, p.w_pre ? x[v] * inv * ((const f32x4 *)p.w_pre)[c] : x[v]);
        }
    } else {
        // any width: the row is worked out again for every pass; a thread reads and writes its own columns only
        auto sum = [&](int c) {
            if (!p.w) return xr[c];
            float t = p.y[(size_t)r * p.ldy + c];
            for (int s = 1; s < p.y_slices; s++) t += p.y[(size_t)s * p.y_stride + (size_t)r * p.ldy + c];
            return fmaf(p.alpha, xr[c], t);
        };
        float inv = 1.0f;
        if (p.w) {
            float ss = 0.f;
            for (int c = tid; c < p.cols; c += nt) {
                const float t = sum(c);
                ss = fmaf(t, t, ss);
            }
            inv = 1.0f / sqrtf(block_sum(ss, sm) / n + p.eps);
        }
        auto result = [&](int c, bool keep) {
            float t = p.w ? sum(c) * inv * p.w[c] : xr[c];
            if (!hr) return t;
            if (keep) hr[(size_t)(p.n_avg - 1) * p.hist_stride + c] = t;
            t *= p.avg[p.n_avg - 1];
            for (int j = 0; j + 1 < p.n_avg; j++) t += p.avg[j] * hr[(size_t)j * p.hist_stride + c];
            return t;
        };
        float inv_o = 1.0f;
        if (out && p.w_pre) {
            float ss = 0.f;
            for (int c = tid; c < p.cols; c += nt) {
                const float t = result(c, false);
                ss = fmaf(t, t, ss);
            }
            inv_o = 1.0f / sqrtf(block_sum(ss, sm) / n + p.eps);
        }
        for (int c = tid; c < p.cols; c += nt) {
            const float t = result(c, p.keep);
            if (xo) xo[c] = t;
            if (out) out[c] = (T)(p.w_pre ? t * inv_o * p.w_pre[c] : t);
        }
    }
    if (out)
        for (int c = p.cols + tid; c < p.ldo; c += nt) out[c] = (T)0.f;
}

// A row's mean and 1 / standard deviation from its columns in registers (zero beyond cols; n4: how many pieces of four there are).
template <int NV>
__device__ __forceinline__ float mean_and_scale(const f32x4 (&v)[NV], int n4, int cols, float eps, float *sm, float *mean) {
    const int tid = threadIdx.x, nt = blockDim.x;
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < NV; i++) t += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
    *mean = block_sum(t, sm) / (float)cols;
    t = 0.f;
#pragma unroll
    for (int i = 0; i < NV; i++)
        if (tid + i * nt < n4)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const float d = v[i][e] - *mean;
                t = fmaf(d, d, t);
            }
    return 1.0f / sqrtf(block_sum(t, sm) / (float)cols + eps);
}

// NV > 0: as for residual_norm_kernel. NV 0: the sublayer's row passes through LDS (cols floats).
template <typename T, int NV>
__global__ void __launch_bounds__(1024) branch_norm_kernel(vx_branch_norm_args p) {
    extern __shared__ float s_row[];
    __shared__ float sm[16];
    const int i = blockIdx.x, r = p.row_idx ? p.row_idx[i] : i, tid = threadIdx.x, nt = blockDim.x;
    const float *xr = p.x_in + (size_t)(p.tokens ? p.tokens[r] : r) * p.cols;
    const float *pr = p.tokens ? p.positions + (size_t)p.token_pos[r] * p.cols : nullptr;
    float *xo = p.x_out ? p.x_out + (size_t)r * p.cols : nullptr;
    T *out = p.out ? (T *)p.out + (size_t)i * p.ldo : nullptr;
    vx_residual_norm_args ex;  // (what add_experts reads)
    ex.e_rows = p.e_rows, ex.lde = p.lde, ex.e_top = p.e_top, ex.e_shared = -1, ex.e_places = p.e_places, ex.e_weights = p.e_weights;
    float mean, inv;
    if constexpr (NV > 0) {
        f32x4 x[NV];
        const int n4 = p.cols >> 2;
        if (p.w) {
            f32x4 y[NV];
#pragma unroll
            for (int v = 0; v < NV; v++) {
                const int c = tid + v * nt;
                y[v] = x[v] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (c >= n4) continue;
                x[v] = ((const f32x4 *)xr)[c];
                if (p.y) {
                    const float *yr = p.y + (size_t)r * p.ldy + c * 4;
                    y[v] = *(const f32x4 *)yr;
                    for (int s = 1; s < p.y_slices; s++) y[v] += *(const f32x4 *)(yr + (size_t)s * p.y_stride);
                    if (p.y_bias) y[v] += ((const f32x4 *)p.y_bias)[c];
                }
                if (p.e_rows) add_experts<T>(ex, r, c * 4, &y[v]);
            }
            inv = mean_and_scale<NV>(y, n4, p.cols, p.eps, sm, &mean);
#pragma unroll
            for (int v = 0; v < NV; v++)
                if (const int c = tid + v * nt; c < n4) x[v] += (y[v] - mean) * inv * ((const f32x4 *)p.w)[c] + ((const f32x4 *)p.b)[c];
        } else {
#pragma unroll
            for (int v = 0; v < NV; v++) {
                const int c = tid + v * nt;
                x[v] = c < n4 ? ((const f32x4 *)xr)[c] : f32x4{0.f, 0.f, 0.f, 0.f};
                if (pr && c < n4) x[v] += ((const f32x4 *)pr)[c];
            }
        }
        const auto keep = [&]() {
#pragma unroll
            for (int v = 0; v < NV; v++)
                if (const int c = tid + v * nt; xo && c < n4) ((f32x4 *)xo)[c] = x[v];
        };
        if (!p.tokens) keep();
        if (p.w_pre) {
            inv = mean_and_scale<NV>(x, n4, p.cols, p.eps, sm, &mean);
#pragma unroll
            for (int v = 0; v < NV; v++)
                if (const int c = tid + v * nt; c < n4) x[v] = (x[v] - mean) * inv * ((const f32x4 *)p.w_pre)[c] + ((const f32x4 *)p.b_pre)[c];
        }
        if (p.tokens) keep();
        if (!out) return;
#pragma unroll
        for (int v = 0; v < NV; v++)
            if (const int c = tid + v * nt; c < n4) store4(out + c * 4, x[v]);
    } else {  // (a thread reads and writes its own columns only)
        const auto norm = [&]() {
            float t = 0.f;
            for (int c = tid; c < p.cols; c += nt) t += s_row[c];
            mean = block_sum(t, sm) / (float)p.cols;
            t = 0.f;
            for (int c = tid; c < p.cols; c += nt) t = fmaf(s_row[c] - mean, s_row[c] - mean, t);
            inv = 1.0f / sqrtf(block_sum(t, sm) / (float)p.cols + p.eps);
        };
        for (int c = tid; c < p.cols; c += nt) {
            float y = 0.f;
            if (p.w) {
                if (p.y) {
                    y = p.y[(size_t)r * p.ldy + c];
                    for (int s = 1; s < p.y_slices; s++) y += p.y[(size_t)s * p.y_stride + (size_t)r * p.ldy + c];
                    if (p.y_bias) y += p.y_bias[c];
                }
                if (p.e_rows) add_experts<T>(ex, r, c, &y);
            } else {
                y = pr ? xr[c] + pr[c] : xr[c];
            }
            s_row[c] = y;
        }
        if (p.w) {
            norm();
            for (int c = tid; c < p.cols; c += nt) s_row[c] = xr[c] + ((s_row[c] - mean) * inv * p.w[c] + p.b[c]);
        }
        if (xo && !p.tokens)
            for (int c = tid; c < p.cols; c += nt) xo[c] = s_row[c];
        if (p.w_pre) {
            norm();
            for (int c = tid; c < p.cols; c += nt) s_row[c] = (s_row[c] - mean) * inv * p.w_pre[c] + p.b_pre[c];
        }
        if (xo && p.tokens)
            for (int c = tid; c < p.cols; c += nt) xo[c] = s_row[c];
        if (!out) return;
        for (int c = tid; c < p.cols; c += nt) out[c] = (T)s_row[c];
    }
    for (int c = p.cols + tid; c < p.ldo; c += nt) out[c] = (T)0.f;
}

// A row per workgroup; NV > 0: cols is a multiple of 8 and at most 8 * NV * blockDim.x, rows aligned: they live in registers.
// Z: bfloat16 or float32, the latter in `slices` parts that are added up.
template <typename T, typename Z, int NV>
__global__ void __launch_bounds__(1024) poly_norm_kernel(const Z *z, int ldz, int slices, int64_t stride, int cols, const float *coef, float eps, T *out,
                                                         int ldo) {
    typedef typename Vec8<T>::type V8;
    typedef typename Vec8<Z>::type Z8;
    __shared__ float sm[3][16];
    const int tid = threadIdx.x, nt = blockDim.x, waves = nt >> 6;
    const Z *zr = z + (size_t)blockIdx.x * ldz;
    T *o = out + (size_t)blockIdx.x * ldo;
    float s[3] = {0.f, 0.f, 0.f};
    const auto add = [&](float t) {
        const float q = t * t;
        s[0] += q;
        s[1] = fmaf(q, q, s[1]);
        s[2] = fmaf(q * q, q, s[2]);
    };
    const auto at = [&](int c) {
        float t = (float)zr[c];
        if constexpr (sizeof(Z) == 4)
            for (int k = 1; k < slices; k++) t += zr[(size_t)k * stride + c];
        return t;
    };
    Z8 v[NV > 0 ? NV : 1];
    if constexpr (NV > 0) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = (tid + i * nt) * 8;
            if (c < cols) v[i] = *(const Z8 *)(zr + c);
            if constexpr (sizeof(Z) == 4)
                for (int k = 1; k < slices; k++)
                    if (c < cols) v[i] += *(const Z8 *)(zr + (size_t)k * stride + c);
        }
#pragma unroll
        for (int i = 0; i < NV; i++)
            if ((tid + i * nt) * 8 < cols)
#pragma unroll
                for (int e = 0; e < 8; e++) add((float)v[i][e]);
    } else {
        for (int c = tid; c < cols; c += nt) add(at(c));
    }
    float f[3];
#pragma unroll
    for (int k = 0; k < 3; k++) {
#pragma unroll
        for (int off = 32; off > 0; off >>= 1) s[k] += __shfl_xor(s[k], off, 64);
        if ((tid & 63) == 0) sm[k][tid >> 6] = s[k];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 3; k++) {
        float t = 0.f;
        for (int w = 0; w < waves; w++) t += sm[k][w];
        f[k] = coef[k] / sqrtf(t / (float)cols + eps);
    }
    const float e0 = coef[3];
    const auto value = [&](float t) { return fmaf(fmaf(fmaf(f[2], t, f[1]), t, f[0]), t, e0); };
    if constexpr (NV > 0) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int c = (tid + i * nt) * 8;
            if (c < cols) {
                V8 w;
#pragma unroll
                for (int e = 0; e < 8; e++) w[e] = (T)value((float)v[i][e]);
                *(V8 *)(o + c) = w;
            }
        }
    } else {
        for (int c = tid; c < cols; c += nt) o[c] = (T)value(at(c));
    }
    for (int c = cols + tid; c < ldo; c += nt) o[c] = (T)0.f;
}

// ---------------------------------------------------------------- convolution
struct ConvArgs {
    vx_conv_args p;
    const int32_t *cu, *pos, *slots;
    int n_seqs, one_token;
};

// A thread takes VEC neighbouring channels of one row.
template <typename T, int VEC>
__global__ void __launch_bounds__(256) conv_silu_kernel(ConvArgs a, int rows) {
    typedef T V __attribute__((ext_vector_type(VEC)));
    typedef float F __attribute__((ext_vector_type(VEC)));
    const vx_conv_args &p = a.p;
    const int per = p.ldo / VEC;
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int row = (int)(id / per), c = (int)(id % per) * VEC;
    if (row >= rows) return;
    V *out = (V *)((T *)p.out + (size_t)row * p.ldo + c);
    if (c >= p.channels) {
        *out = (V)(T)0.f;
        return;
    }
    const int seq = a.one_token ? row : seq_of_row(a.cu, a.n_seqs, row);
    const int local = a.one_token ? 0 : row - a.cu[seq], pos = a.pos[row], hist = p.taps - 1;
    T *st = (T *)p.state + (size_t)a.slots[seq] * hist * p.channels + c;
    const T *x = (const T *)p.x + (size_t)row * p.ldx + c;
    F acc = *(const F *)(p.b + c);
    for (int t = 0; t < p.taps; t++) {
        const int d = hist - t;  // tokens back
        V v = (V)(T)0.f;
        if (d <= local)
            v = *(const V *)(x - (ptrdiff_t)d * p.ldx);
        else if (d <= pos)
            v = *(const V *)(st + (size_t)(hist - (d - local)) * p.channels);
        const F w = *(const F *)(p.w + (size_t)t * p.channels + c);
#pragma unroll
        for (int e = 0; e < VEC; e++) acc[e] = fmaf(w[e], (float)v[e], acc[e]);
    }
    V o;
#pragma unroll
    for (int e = 0; e < VEC; e++) o[e] = (T)silu_f(acc[e]);
    *out = o;
    if (a.one_token) {  // this thread alone reads and moves the channels' history
        for (int k = 0; k + 1 < hist; k++)
            *(V *)(st + (size_t)k * p.channels) = pos - (hist - 1 - k) >= 0 ? *(const V *)(st + (size_t)(k + 1) * p.channels) : (V)(T)0.f;
        if (hist > 0) *(V *)(st + (size_t)(hist - 1) * p.channels) = *(const V *)x;
    }
}

// The history after the step: entry k is the input of position end - (taps - 1 - k), end = the sequence's length.
template <typename T>
__global__ void __launch_bounds__(256) conv_state_kernel(ConvArgs a) {
    const vx_conv_args &p = a.p;
    const int seq = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= p.channels) return;
    const int r0 = a.cu[seq], len = a.cu[seq + 1] - r0, hist = p.taps - 1, start = a.pos[r0];
    T *st = (T *)p.state + (size_t)a.slots[seq] * hist * p.channels + c;
    const T *x = (const T *)p.x + (size_t)r0 * p.ldx + c;
    for (int k = 0; k < hist; k++) {  // ascending: entry k + len is read before it is written
        const int local = len - (hist - k);
        T v = (T)0.f;
        if (local >= 0)
            v = x[(size_t)local * p.ldx];
        else if (start + local >= 0)
            v = st[(size_t)(k + len) * p.channels];
        st[(size_t)k * p.channels] = v;
    }
}

// ---------------------------------------------------------------- scan
constexpr int CHUNK = 64;
constexpr int NS = 8;  // states of a lane

struct ScanArgs {
    vx_scan_args p;
    int pad;
    const int32_t *cu, *pos, *slots;
    int n_seqs, one_token, stage;  // stage: rows of bc staged in LDS at a time
    float *h;     // [chunks][channels][pad]: a chunk's own contribution, then the state before it
    float *sdt;   // [chunks][channels]: sum of dt
};

__device__ __forceinline__ f32x8 load8(const float *p) {
    const f32x4 a = *(const f32x4 *)p, b = *(const f32x4 *)(p + 4);
    return f32x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
__device__ __forceinline__ void store8(float *p, f32x8 v) {
    *(f32x4 *)p = f32x4{v[0], v[1], v[2], v[3]};
    *(f32x4 *)(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}

// FINAL false: the contribution of every chunk that is not its sequence's last; true: outputs, and the final state.
template <typename T, int LP, bool FINAL>
__global__ void __launch_bounds__(256) scan_kernel(ScanArgs a) {
    extern __shared__ float s_bc[];
    const vx_scan_args &p = a.p;
    constexpr int CH = 256 / LP;
    const int sub = threadIdx.x % LP, c = blockIdx.y * CH + threadIdx.x / LP, pad = LP * NS;
    const bool live = c < p.channels;
    const int cc = live ? c : p.channels - 1;
    int seq = blockIdx.x, ci = 0, chunks = 1, len = 1, row0 = blockIdx.x;
    if (!a.one_token) {
        if (!item_of_seq(a.cu, a.n_seqs, CHUNK, 1, blockIdx.x, &seq, &ci, &chunks)) return;
        if (!FINAL && ci + 1 == chunks) return;
        row0 = a.cu[seq] + ci * CHUNK;
        len = min(CHUNK, a.cu[seq + 1] - row0);
    }
    const int slot = a.slots[seq], pos0 = a.pos[row0];
    const size_t sidx = ((size_t)slot * p.channels + cc) * pad + sub * NS;
    const size_t hidx = ((size_t)blockIdx.x * p.channels + cc) * pad + sub * NS;
    f32x8 S = f32x8{0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (FINAL) {
        if (chunks > 1)
            S = load8(a.h + hidx);
        else if (pos0 > 0)
            S = load8(p.state + sidx);
    }
    const f32x8 A = load8(p.a2 + (size_t)cc * pad + sub * NS);
    const float D = p.d[cc];
    float sum = 0.f;
    const float *dt = p.dt + (size_t)row0 * p.lddt + cc;
    const T *x = (const T *)p.x + (size_t)row0 * p.ldx + cc;
    const T *z = FINAL ? (const T *)p.z + (size_t)row0 * p.ldz + cc : nullptr;
    T *out = FINAL ? (T *)p.out + (size_t)row0 * p.ldo + c : nullptr;
    for (int t0 = 0; t0 < len; t0 += a.stage) {
        const int tn = min(a.stage, len - t0);
        __syncthreads();
        const f32x4 *src = (const f32x4 *)(p.bc + (size_t)(row0 + t0) * 2 * pad);
        for (int i = threadIdx.x; i < tn * 2 * pad / 4; i += 256) ((f32x4 *)s_bc)[i] = src[i];
        __syncthreads();
        constexpr int U = 4;
        float ndt[U], nx[U], nz[U];
        auto fetch = [&](int t) {
#pragma unroll
            for (int u = 0; u < U; u++) {
                const int tt = t0 + min(t + u, tn - 1);
                ndt[u] = dt[(size_t)tt * p.lddt];
                nx[u] = (float)x[(size_t)tt * p.ldx];
                if (FINAL) nz[u] = (float)z[(size_t)tt * p.ldz];
            }
        };
        fetch(0);
        for (int t = 0; t < tn; t += U) {
            float cdt[U], cx[U], cz[U];
#pragma unroll
            for (int u = 0; u < U; u++) cdt[u] = ndt[u], cx[u] = nx[u], cz[u] = FINAL ? nz[u] : 0.f;
            if (t + U < tn) fetch(t + U);
#pragma unroll
            for (int u = 0; u < U; u++) {
                if (t + u >= tn) break;
                const float *b = s_bc + (size_t)(t + u) * 2 * pad + sub * NS;
                const f32x8 B = load8(b);
                const float dx = cdt[u] * cx[u];
#pragma unroll
                for (int n = 0; n < NS; n++) S[n] = fmaf(__builtin_amdgcn_exp2f(cdt[u] * A[n]), S[n], dx * B[n]);
                if (FINAL) {
                    const f32x8 C = load8(b + pad);
                    float y = 0.f;
#pragma unroll
                    for (int n = 0; n < NS; n++) y = fmaf(S[n], C[n], y);
#pragma unroll
                    for (int off = LP / 2; off > 0; off >>= 1) y += __shfl_xor(y, off, 64);
                    if (sub == 0 && live)
                        out[(size_t)(t0 + t + u) * p.ldo] = (T)(p.out_scale * (fmaf(D, cx[u], y) * silu_f(cz[u])));
                } else {
                    sum += cdt[u];
                }
            }
        }
    }
    if (FINAL) {
        if (live && ci + 1 == chunks) store8(p.state + sidx, S);
        // the columns that pad the row
        if (blockIdx.y == 0)
            for (int i = threadIdx.x; i < (p.out_cols - p.channels) * len; i += 256) {
                const int w = p.out_cols - p.channels;
                ((T *)p.out)[(size_t)(row0 + i / w) * p.ldo + p.channels + i % w] = (T)0.f;
            }
    } else if (live) {
        store8(a.h + hidx, S);
        if (sub == 0) a.sdt[(size_t)blockIdx.x * p.channels + c] = sum;
    }
}

// Chunk contributions -> the state before every chunk, for sequences with several. One thread per (channel, state).
__global__ void __launch_bounds__(256) scan_carry_kernel(ScanArgs a) {
    const vx_scan_args &p = a.p;
    const int seq = blockIdx.x;
    const size_t e = (size_t)blockIdx.y * 256 + threadIdx.x, per = (size_t)p.channels * a.pad;
    const int chunks = (a.cu[seq + 1] - a.cu[seq] + CHUNK - 1) / CHUNK;
    if (chunks < 2 || e >= per) return;
    int first = 0;
    for (int s = 0; s < seq; s++) first += (a.cu[s + 1] - a.cu[s] + CHUNK - 1) / CHUNK;
    const int c = (int)(e / a.pad);
    const float A = p.a2[e];
    float S = a.pos[a.cu[seq]] > 0 ? p.state[(size_t)a.slots[seq] * per + e] : 0.f;
    constexpr int U = 4;
    for (int k = 0; k < chunks; k += U) {
        float own[U], sd[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int kk = first + min(k + u, chunks - 1);
            own[u] = a.h[(size_t)kk * per + e];
            sd[u] = a.sdt[(size_t)kk * p.channels + c];
        }
#pragma unroll
        for (int u = 0; u < U; u++) {
            if (k + u >= chunks) break;
            a.h[(size_t)(first + k + u) * per + e] = S;
            S = fmaf(__builtin_amdgcn_exp2f(sd[u] * A), S, own[u]);  // (after the last chunk: not used)
        }
    }
}

template <typename T, int LP>
void launch_scan(vx_backend *be, const ScanArgs &a, int chunks, bool several) {
    const dim3 grid(chunks, ceil_div(a.p.channels, 256 / LP));
    const size_t lds = (size_t)a.stage * 2 * a.pad * sizeof(float);
    if (several) {
        scan_kernel<T, LP, false><<<grid, 256, lds, be->stream>>>(a);
        const size_t per = (size_t)a.p.channels * a.pad;
        scan_carry_kernel<<<dim3(a.n_seqs, (unsigned)ceil_div64((int64_t)per, 256)), 256, 0, be->stream>>>(a);
    }
    scan_kernel<T, LP, true><<<grid, 256, lds, be->stream>>>(a);
}

template <typename T>
void dispatch_scan(vx_backend *be, const ScanArgs &a, int chunks, bool several) {
    switch (a.pad / NS) {
        case 2: launch_scan<T, 2>(be, a, chunks, several); break;
        case 4: launch_scan<T, 4>(be, a, chunks, several); break;
        case 8: launch_scan<T, 8>(be, a, chunks, several); break;
        case 16: launch_scan<T, 16>(be, a, chunks, several); break;
        default: launch_scan<T, 32>(be, a, chunks, several); break;
    }
}

template <typename T>
void launch_norm(vx_backend *be, const vx_residual_norm_args &p) {
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = p.cols % 4 == 0 && al(p.x_in) && al(p.add) && al(p.x_out) && al(p.y) && al(p.w_post) && al(p.w_pre) &&
                     al(p.out) && al(p.y_bias) && al(p.e_rows) && (!p.e_rows || p.lde % 4 == 0) && (!p.y || (p.ldy % 4 == 0 && p.y_stride % 4 == 0)) && (!p.w_pre || p.ldo % 4 == 0);
    const int n4 = p.cols / 4;
    // few rows: many threads each, so that a decode step's rows are short
    int threads = p.rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads / 2 >= n4) threads /= 2;
    const int nv = ceil_div(n4, threads);
    if (!vec || nv > 8)
        residual_norm_kernel<T, 0><<<p.rows, 256, 0, be->stream>>>(p);
    else if (nv <= 1)
        residual_norm_kernel<T, 1><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 2)
        residual_norm_kernel<T, 2><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 4)
        residual_norm_kernel<T, 4><<<p.rows, threads, 0, be->stream>>>(p);
    else
        residual_norm_kernel<T, 8><<<p.rows, threads, 0, be->stream>>>(p);
}

template <typename T>
void launch_post_norm(vx_backend *be, const vx_post_norm_args &p) {
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = p.cols % 4 == 0 && al(p.x_in) && al(p.x_out) && al(p.y) && al(p.w) && al(p.w_pre) && al(p.out) && al(p.hist) &&
                     p.hist_stride % 4 == 0 && (!p.w || (p.ldy % 4 == 0 && p.y_stride % 4 == 0)) && p.ldo % 4 == 0;
    const int n4 = p.cols / 4;
    int threads = p.rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads / 2 >= n4) threads /= 2;
    const int nv = ceil_div(n4, threads);
    if (!vec || nv > 8)
        post_norm_kernel<T, 0><<<p.rows, 256, 0, be->stream>>>(p);
    else if (nv <= 1)
        post_norm_kernel<T, 1><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 2)
        post_norm_kernel<T, 2><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 4)
        post_norm_kernel<T, 4><<<p.rows, threads, 0, be->stream>>>(p);
    else
        post_norm_kernel<T, 8><<<p.rows, threads, 0, be->stream>>>(p);
}

template <typename T>
void launch_branch_norm(vx_backend *be, const vx_branch_norm_args &p) {
    const auto al = [](const void *q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = p.cols % 4 == 0 && al(p.x_in) && al(p.x_out) && al(p.y) && al(p.y_bias) && al(p.w) && al(p.b) && al(p.w_pre) && al(p.b_pre) && al(p.out) &&
                     al(p.positions) && al(p.e_rows) && (!p.e_rows || p.lde % 4 == 0) && (!p.y || (p.ldy % 4 == 0 && p.y_stride % 4 == 0)) &&
                     (!p.out || p.ldo % 4 == 0);
    const int n4 = p.cols / 4;
    int threads = p.rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads / 2 >= n4) threads /= 2;
    while (threads < 1024 && n4 > 8 * threads) threads *= 2;
    const int nv = ceil_div(n4, threads);
    if (!vec || nv > 8)
        branch_norm_kernel<T, 0><<<p.rows, 256, (size_t)p.cols * 4, be->stream>>>(p);
    else if (nv <= 1)
        branch_norm_kernel<T, 1><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 2)
        branch_norm_kernel<T, 2><<<p.rows, threads, 0, be->stream>>>(p);
    else if (nv <= 4)
        branch_norm_kernel<T, 4><<<p.rows, threads, 0, be->stream>>>(p);
    else
        branch_norm_kernel<T, 8><<<p.rows, threads, 0, be->stream>>>(p);
}

template <typename T, typename Z>
void launch_poly_norm(vx_backend *be, const Z *z, int ldz, int slices, int64_t stride, int rows, int cols, const float *coef, float eps, T *out, int ldo) {
    const bool vec = cols % 8 == 0 && ldz % 8 == 0 && ldo % 8 == 0 && (slices == 1 || stride % 8 == 0) && (uintptr_t)z % 16 == 0 && (uintptr_t)out % 16 == 0;
    const int n8 = cols / 8;
    int threads = rows <= 256 ? 1024 : 256;
    while (threads > 64 && threads / 2 >= n8) threads /= 2;
    while (threads < 1024 && n8 > 4 * threads) threads *= 2;
    const int nv = ceil_div(n8, threads);
    if (!vec || nv > 4)
        poly_norm_kernel<T, Z, 0><<<rows, 1024, 0, be->stream>>>(z, ldz, slices, stride, cols, coef, eps, out, ldo);
    else if (nv <= 1)
        poly_norm_kernel<T, Z, 1><<<rows, threads, 0, be->stream>>>(z, ldz, slices, stride, cols, coef, eps, out, ldo);
    else if (nv <= 2)
        poly_norm_kernel<T, Z, 2><<<rows, threads, 0, be->stream>>>(z, ldz, slices, stride, cols, coef, eps, out, ldo);
    else
        poly_norm_kernel<T, Z, 4><<<rows, threads, 0, be->stream>>>(z, ldz, slices, stride, cols, coef, eps, out, ldo);
}

}  // namespace

extern "C" {

int vx_post_norm(vx_backend *be, int act, const vx_post_norm_args *a) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(a && a->rows >= 1 && a->cols >= 1 && a->x_in, "vx_post_norm: bad arguments");
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_post_norm: unknown activation type %d", act);
    VX_REQUIRE(!a->w || (a->y && a->y_slices >= 1 && a->ldy >= a->cols), "vx_post_norm: incomplete sublayer output");
    VX_REQUIRE(a->n_avg == 0 || (a->n_avg > 0 && a->hist && a->avg && a->hist_stride >= 0), "vx_post_norm: incomplete average");
    VX_REQUIRE(!a->out || a->ldo >= a->cols, "vx_post_norm: rows of %d for %d columns", a->ldo, a->cols);
    VX_REQUIRE(a->out || a->x_out, "vx_post_norm: nothing to write");
    if (act == VX_ACT_BF16)
        launch_post_norm<bf16>(be, *a);
    else
        launch_post_norm<float>(be, *a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_branch_norm(vx_backend *be, int act, const vx_branch_norm_args *a) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(a && a->rows >= 1 && a->cols >= 1 && a->x_in, "vx_branch_norm: bad arguments");
    VX_REQUIRE(a->cols <= 15360 || a->cols % 4 == 0, "vx_branch_norm: rows of %d columns", a->cols);
    VX_REQUIRE(a->cols <= 32768, "vx_branch_norm: rows of %d columns", a->cols);
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_branch_norm: unknown activation type %d", act);
    VX_REQUIRE(!a->w || (a->b && (a->y || a->e_rows)), "vx_branch_norm: incomplete norm");
    VX_REQUIRE(!a->y || (a->y_slices >= 1 && a->ldy >= a->cols), "vx_branch_norm: incomplete sublayer output");
    VX_REQUIRE(!a->e_rows || (a->lde >= a->cols && a->e_top >= 1 && a->e_places && a->e_weights), "vx_branch_norm: incomplete experts");
    VX_REQUIRE(!a->w_pre || a->b_pre, "vx_branch_norm: incomplete norm of the result");
    VX_REQUIRE(!a->tokens || (!a->w && !a->row_idx && a->token_pos && a->positions && a->w_pre), "vx_branch_norm: incomplete embedding");
    VX_REQUIRE(!a->out || a->ldo >= a->cols, "vx_branch_norm: rows of %d for %d columns", a->ldo, a->cols);
    VX_REQUIRE(a->out || a->x_out, "vx_branch_norm: nothing to write");
    if (act == VX_ACT_BF16)
        launch_branch_norm<bf16>(be, *a);
    else
        launch_branch_norm<float>(be, *a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_poly_norm(vx_backend *be, int act, const void *z, int ldz, int z_slices, int64_t z_stride, int rows, int cols, const float *coef, float eps,
                 void *out, int ldo) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_poly_norm: unknown activation type %d", act);
    VX_REQUIRE(z && coef && out && z != out && rows >= 1 && cols >= 1 && ldz >= cols && ldo >= cols && z_slices >= 0, "vx_poly_norm: bad arguments");
    if (act == VX_ACT_F32)
        launch_poly_norm<float, float>(be, (const float *)z, ldz, z_slices > 1 ? z_slices : 1, z_stride, rows, cols, coef, eps, (float *)out, ldo);
    else if (z_slices > 0)
        launch_poly_norm<bf16, float>(be, (const float *)z, ldz, z_slices, z_stride, rows, cols, coef, eps, (bf16 *)out, ldo);
    else
        launch_poly_norm<bf16, bf16>(be, (const bf16 *)z, ldz, 1, 0, rows, cols, coef, eps, (bf16 *)out, ldo);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_residual_norm(vx_backend *be, int act, const vx_residual_norm_args *a) {
    int rc = enter(be);
    if (rc) return rc;
    VX_REQUIRE(a && a->rows >= 1 && a->cols >= 1 && a->x_in, "vx_residual_norm: bad arguments");
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_residual_norm: unknown activation type %d", act);
    VX_REQUIRE(!a->y || (a->y_slices >= 1 && a->ldy >= a->cols && !(a->w_post && a->y_bias)), "vx_residual_norm: incomplete sublayer output");
    VX_REQUIRE(!a->e_rows || (a->lde >= a->cols && a->e_top >= 0 && (a->e_top == 0 || (a->e_places && a->e_weights))), "vx_residual_norm: incomplete experts");
    VX_REQUIRE(!a->w_pre || (a->out && a->ldo >= a->cols), "vx_residual_norm: incomplete output");
    VX_REQUIRE(a->w_pre || a->x_out, "vx_residual_norm: nothing to write");
    if (act == VX_ACT_BF16)
        launch_norm<bf16>(be, *a);
    else
        launch_norm<float>(be, *a);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_conv_silu(vx_backend *be, int act, const vx_ragged *b, const vx_conv_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_conv_silu");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_conv_silu: unknown activation type %d", act);
    VX_REQUIRE(p && p->channels >= 1 && p->taps >= 1 && p->x && p->w && p->b && p->out && (p->state || p->taps == 1) &&
                   p->ldx >= p->channels && p->ldo >= p->channels,
               "vx_conv_silu: bad arguments");
    ConvArgs a{*p, b->cu_seqlens, b->token_pos, b->table_rows, b->n_seqs, b->q_lens ? 0 : 1};
    const auto al = [](const void *q) { return (uintptr_t)q % 32 == 0; };
    const bool vec = p->channels % 8 == 0 && p->ldx % 8 == 0 && p->ldo % 8 == 0 && al(p->w) && al(p->b) && (uintptr_t)p->x % 16 == 0 &&
                     (uintptr_t)p->out % 16 == 0 && (uintptr_t)p->state % 16 == 0 && act == VX_ACT_BF16;
    const unsigned grid = (unsigned)ceil_div64((int64_t)b->rows * (p->ldo / (vec ? 8 : 1)), 256);
    const dim3 sgrid(b->n_seqs, ceil_div(p->channels, 256));
    if (vec)
        conv_silu_kernel<bf16, 8><<<grid, 256, 0, be->stream>>>(a, b->rows);
    else if (act == VX_ACT_BF16)
        conv_silu_kernel<bf16, 1><<<grid, 256, 0, be->stream>>>(a, b->rows);
    else
        conv_silu_kernel<float, 1><<<grid, 256, 0, be->stream>>>(a, b->rows);
    if (b->q_lens && p->taps > 1) {
        if (act == VX_ACT_BF16)
            conv_state_kernel<bf16><<<sgrid, 256, 0, be->stream>>>(a);
        else
            conv_state_kernel<float><<<sgrid, 256, 0, be->stream>>>(a);
    }
    VX_CHECK_LAUNCH();
    return VX_OK;
}

int vx_scan_state_pad(int states) {
    if (states < 1 || states > 256) return -1;
    int pad = 2 * NS;
    while (pad < states) pad *= 2;
    return pad;
}

int vx_selective_scan(vx_backend *be, int act, const vx_ragged *b, const vx_scan_args *p) {
    int rc = enter(be);
    if (rc) return rc;
    rc = check_ragged(b, "vx_selective_scan");
    if (rc) return rc;
    VX_REQUIRE(act == VX_ACT_F32 || act == VX_ACT_BF16, "vx_selective_scan: unknown activation type %d", act);
    VX_REQUIRE(p && p->channels >= 1 && p->a2 && p->d && p->x && p->z && p->dt && p->bc && p->state && p->out,
               "vx_selective_scan: null argument");
    const int pad = vx_scan_state_pad(p->states);
    VX_REQUIRE(pad > 0, "vx_selective_scan: %d states not in 1..256", p->states);
    VX_REQUIRE(p->ldx >= p->channels && p->ldz >= p->channels && p->lddt >= p->channels && p->out_cols >= p->channels &&
                   p->ldo >= p->out_cols && (uintptr_t)p->bc % 16 == 0 && (uintptr_t)p->a2 % 16 == 0 && (uintptr_t)p->state % 16 == 0,
               "vx_selective_scan: bad strides");
    ScanArgs a{*p, pad, b->cu_seqlens, b->token_pos, b->table_rows, b->n_seqs, b->q_lens ? 0 : 1, 0, nullptr, nullptr};
    a.stage = 8192 / pad < CHUNK ? 8192 / pad : CHUNK;  // at most 64 KB of LDS
    if (!b->q_lens) a.stage = 1;
    const int chunks = count_items(b, CHUNK, 1);
    const bool several = chunks > b->n_seqs;
    if (several) {
        const size_t h = (size_t)chunks * p->channels * pad * sizeof(float), sd = (size_t)chunks * p->channels * sizeof(float);
        rc = ensure_ws(be, &be->scan_ws, &be->scan_ws_bytes, h + sd, "scan");
        if (rc) return rc;
        a.h = (float *)be->scan_ws;
        a.sdt = (float *)((char *)be->scan_ws + h);
    }
    if (act == VX_ACT_BF16)
        dispatch_scan<bf16>(be, a, chunks, several);
    else
        dispatch_scan<float>(be, a, chunks, several);
    VX_CHECK_LAUNCH();
    return VX_OK;
}

}  // extern "C"
