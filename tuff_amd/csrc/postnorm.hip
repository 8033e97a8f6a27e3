// Kernels of layers that norm a sublayer's output before it joins the residual stream, all in float32.
//
// tuff_post_norm_add, a workgroup a token:
//     x <- x + mult * y / sqrt(mean(y^2) + eps) * w  [+ extra] [+ row]   (y is then cleared, if asked, or set to a row
//                                                                      y_next: the bias of the product that adds into y next)
//     h  = x / sqrt(mean(x^2) + eps_next) * w_next                     (if asked: the next sublayer's input; without a
//                                                                      weight h is x itself, rounded to its type)
// y may lack a bias, a row y_bias that is added to it before anything else.
// One launch where a norm, a residual sum, another sum and the next norm would be four.  Without y only the
// sum with `extra` and the next norm run.  The weights come in as float32 with any offset already added.
//
// tuff_normed_mean2, a workgroup a token:
//     out <- out + coef * (a / sqrt(mean(a^2) + eps) * wa + b / sqrt(mean(b^2) + eps) * wb)
// for a mixer made of two mixers side by side whose outputs are each normed over the width.
//
// tuff_scale_add_layer_norm, a workgroup a token, for layers that scale a sublayer's output per channel:
//     x <- x + ls * y                                                   (y is then cleared, if asked)
//     h  = (x - mean(x)) / sqrt(mean((x - mean(x))^2) + eps) * w_next   (if asked: the next sublayer's input)
// a layer norm with a weight and no bias, the variance taken from the deviations themselves.  Without y the norm
// alone runs, then optionally over chosen rows of x only (the rows whose logits are wanted).
//
// Every row's sums run over the row in one fixed order (a thread's elements in ascending order, the
// butterfly of a wave, the waves in order), so a row's result does not depend on what else is in the step.
#include "common.h"
#include <math.h>

namespace {
constexpr int PN_THREADS = 256;
constexpr int PN_WAVES = PN_THREADS / WAVE;

template <typename T>
__global__ __launch_bounds__(PN_THREADS) void post_norm_add_kernel(
    float* __restrict__ x, float* __restrict__ y, const float* __restrict__ w, float eps, float mult,
    const float* __restrict__ extra, const float* __restrict__ w_next, float eps_next, T* __restrict__ h_out,
    int d, int clear_y, const float* __restrict__ y_next, const float* __restrict__ y_bias, const float* __restrict__ row_add) {
    __shared__ float scratch[PN_WAVES];
    const long long row = (long long)blockIdx.x * d;
    float* xr = x + row;
    float inv = 0.f;
    if (y) {
        const float* yr = y + row;
        float ss = 0.f;
        for (int c = threadIdx.x; c < d; c += PN_THREADS) {
            const float v = y_bias ? yr[c] + y_bias[c] : yr[c];
            ss = fmaf(v, v, ss);
        }
        ss = block_sum<PN_WAVES>(ss, scratch);
        inv = mult / sqrtf(ss / (float)d + eps);
    }
    float ss2 = 0.f;
    for (int c = threadIdx.x; c < d; c += PN_THREADS) {
        float v = xr[c];
        if (y) {
            v = fmaf((y_bias ? y[row + c] + y_bias[c] : y[row + c]) * inv, w[c], v);
            if (clear_y) y[row + c] = y_next ? y_next[c] : 0.f;
        }
        if (extra) v += extra[row + c];
        if (row_add) v += row_add[c];
        if (y || extra || row_add) xr[c] = v;
        ss2 = fmaf(v, v, ss2);
    }
    if (!h_out) return;
    if (!w_next) {
        for (int c = threadIdx.x; c < d; c += PN_THREADS) h_out[row + c] = from_f32<T>(xr[c]);
        return;
    }
    ss2 = block_sum<PN_WAVES>(ss2, scratch);
    const float inv2 = 1.0f / sqrtf(ss2 / (float)d + eps_next);
    // (a thread reads back the elements it wrote itself)
    for (int c = threadIdx.x; c < d; c += PN_THREADS) h_out[row + c] = from_f32<T>(xr[c] * inv2 * w_next[c]);
}

// The same for rows of at most PN_THREADS * EPT elements: a thread keeps its elements in registers, and everything a
// row needs is loaded before the first sum, so the launch waits for memory once.  The sums run in the order of the
// kernel above (a thread's elements in ascending order): the same bits.
template <typename T, int EPT>
__global__ __launch_bounds__(PN_THREADS) void post_norm_add_regs_kernel(
    float* __restrict__ x, float* __restrict__ y, const float* __restrict__ w, float eps, float mult,
    const float* __restrict__ extra, const float* __restrict__ w_next, float eps_next, T* __restrict__ h_out,
    int d, int clear_y, const float* __restrict__ y_next, const float* __restrict__ y_bias, const float* __restrict__ row_add) {
    __shared__ float scratch[PN_WAVES];
    const long long row = (long long)blockIdx.x * d;
    float xv[EPT], yv[EPT], wv[EPT], ev[EPT], rv[EPT], nv[EPT];
#pragma unroll
    for (int k = 0; k < EPT; ++k) {
        const int c = threadIdx.x + k * PN_THREADS;
        const bool in = c < d;
        xv[k] = in ? x[row + c] : 0.f;
        yv[k] = (in && y) ? y[row + c] : 0.f;
        if (y_bias && in) yv[k] += y_bias[c];
        wv[k] = (in && y) ? w[c] : 0.f;
        ev[k] = (in && extra) ? extra[row + c] : 0.f;
        rv[k] = (in && row_add) ? row_add[c] : 0.f;
        nv[k] = (in && w_next) ? w_next[c] : 0.f;
    }
    float inv = 0.f;
    if (y) {
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < EPT; ++k)
            if (threadIdx.x + k * PN_THREADS < d) ss = fmaf(yv[k], yv[k], ss);
        ss = block_sum<PN_WAVES>(ss, scratch);
        inv = mult / sqrtf(ss / (float)d + eps);
    }
    float ss2 = 0.f;
#pragma unroll
    for (int k = 0; k < EPT; ++k) {
        const int c = threadIdx.x + k * PN_THREADS;
        if (c >= d) continue;
        float v = xv[k];
        if (y) {
            v = fmaf(yv[k] * inv, wv[k], v);
            if (clear_y) y[row + c] = y_next ? y_next[c] : 0.f;
        }
        if (extra) v += ev[k];
        if (row_add) v += rv[k];
        if (y || extra || row_add) x[row + c] = v;
        xv[k] = v;
        ss2 = fmaf(v, v, ss2);
    }
    if (!h_out) return;
    if (!w_next) {
#pragma unroll
        for (int k = 0; k < EPT; ++k) {
            const int c = threadIdx.x + k * PN_THREADS;
            if (c < d) h_out[row + c] = from_f32<T>(xv[k]);
        }
        return;
    }
    ss2 = block_sum<PN_WAVES>(ss2, scratch);
    const float inv2 = 1.0f / sqrtf(ss2 / (float)d + eps_next);
#pragma unroll
    for (int k = 0; k < EPT; ++k) {
        const int c = threadIdx.x + k * PN_THREADS;
        if (c < d) h_out[row + c] = from_f32<T>(xv[k] * inv2 * nv[k]);
    }
}

// The same for rows of a multiple of four elements, up to 4,096: a thread holds VPT times four neighbouring ones, a workgroup
// has as many waves as the row needs, so a row's few loads are 16 bytes wide and all under way at once, which is what a step
// of few tokens waits for.  Sums: a thread's elements in ascending order, the butterfly of a wave, the waves in order.
constexpr int PN_VEC_MAX = 4096;

__device__ __forceinline__ float waves_sum(float v, float* scratch, int waves) {
    v = wave_sum(v);
    if (threadIdx.x % WAVE == 0) scratch[threadIdx.x / WAVE] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < waves; ++i) t += scratch[i];
    return t;
}

template <typename T, int VPT>
__global__ __launch_bounds__(PN_VEC_MAX / 4 / VPT) void post_norm_add_vec_kernel(
    float* __restrict__ x, float* __restrict__ y, const float* __restrict__ w, float eps, float mult,
    const float* __restrict__ extra, const float* __restrict__ w_next, float eps_next, T* __restrict__ h_out,
    int d, int clear_y, const float* __restrict__ y_next, const float* __restrict__ y_bias, const float* __restrict__ row_add) {
    typedef T out4 __attribute__((ext_vector_type(4)));
    __shared__ float scratch[2][PN_VEC_MAX / 4 / WAVE];
    const int waves = blockDim.x / WAVE;
    const long long row = (long long)blockIdx.x * d;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    f32x4 xv[VPT], yv[VPT], wv[VPT], ev[VPT], rv[VPT], nv[VPT];
    auto place = [&](int k) { return (int)(threadIdx.x + k * blockDim.x) * 4; };
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int c = place(k);
        const bool in = c < d;
        xv[k] = in ? *(const f32x4*)(x + row + c) : zero;
        yv[k] = (in && y) ? *(const f32x4*)(y + row + c) : zero;
        wv[k] = (in && y) ? *(const f32x4*)(w + c) : zero;
        if (in && y_bias) yv[k] += *(const f32x4*)(y_bias + c);
        ev[k] = (in && extra) ? *(const f32x4*)(extra + row + c) : zero;
        rv[k] = (in && row_add) ? *(const f32x4*)(row_add + c) : zero;
        nv[k] = (in && w_next) ? *(const f32x4*)(w_next + c) : zero;
    }
    if (y) {
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k)
#pragma unroll
            for (int e = 0; e < 4; ++e) ss = fmaf(yv[k][e], yv[k][e], ss);
        ss = waves_sum(ss, scratch[0], waves);
        const float inv = mult / sqrtf(ss / (float)d + eps);
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int c = place(k);
#pragma unroll
            for (int e = 0; e < 4; ++e) xv[k][e] = fmaf(yv[k][e] * inv, wv[k][e], xv[k][e]);
            if (c < d && clear_y) *(f32x4*)(y + row + c) = y_next ? *(const f32x4*)(y_next + c) : zero;
        }
    }
    float ss2 = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int c = place(k);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            if (extra) xv[k][e] += ev[k][e];
            if (row_add) xv[k][e] += rv[k][e];
            ss2 = fmaf(xv[k][e], xv[k][e], ss2);
        }
        if (c < d && (y || extra || row_add)) *(f32x4*)(x + row + c) = xv[k];
    }
    if (!h_out) return;
    float inv2 = 1.0f;
    if (w_next) inv2 = 1.0f / sqrtf(waves_sum(ss2, scratch[1], waves) / (float)d + eps_next);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int c = place(k);
        out4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = from_f32<T>(w_next ? xv[k][e] * inv2 * nv[k][e] : xv[k][e]);
        if (c < d) *(out4*)(h_out + row + c) = o;
    }
}

__global__ __launch_bounds__(PN_THREADS) void normed_mean2_kernel(
    const float* __restrict__ a, const float* __restrict__ wa, const float* __restrict__ b, const float* __restrict__ wb,
    float eps, float coef, float* __restrict__ out, int d) {
    __shared__ float scratch[PN_WAVES];
    const long long row = (long long)blockIdx.x * d;
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x; c < d; c += PN_THREADS) {
        sa = fmaf(a[row + c], a[row + c], sa);
        sb = fmaf(b[row + c], b[row + c], sb);
    }
    sa = block_sum<PN_WAVES>(sa, scratch);
    sb = block_sum<PN_WAVES>(sb, scratch);
    const float ia = 1.0f / sqrtf(sa / (float)d + eps), ib = 1.0f / sqrtf(sb / (float)d + eps);
    for (int c = threadIdx.x; c < d; c += PN_THREADS)
        out[row + c] += coef * (a[row + c] * ia * wa[c] + b[row + c] * ib * wb[c]);
}

// EPT > 0: rows of at most PN_THREADS * EPT elements stay in registers between the sums; EPT 0: any width, the row
// read again from x for every pass (a thread reads back what it wrote itself).  The sums run in the same order.
template <typename T, int EPT>
__global__ __launch_bounds__(PN_THREADS) void scale_add_layer_norm_kernel(
    float* __restrict__ x, float* __restrict__ y, const float* __restrict__ ls, const float* __restrict__ w_next, float eps,
    T* __restrict__ h_out, const int* __restrict__ rows, int d, int clear_y) {
    __shared__ float scratch[PN_WAVES];
    const long long src = (long long)(rows ? rows[blockIdx.x] : (int)blockIdx.x) * d;
    const long long dst = (long long)blockIdx.x * d;
    constexpr int N = EPT > 0 ? EPT : 1;
    float xv[N];
    float sum = 0.f;
    float nv[N];                                       // the next norm's weight: asked for with everything else, before the first sum
    if (EPT > 0) {
        float yv[N], lv[N];
#pragma unroll
        for (int k = 0; k < N; ++k) {
            const int c = threadIdx.x + k * PN_THREADS;
            const bool in = c < d;
            xv[k] = in ? x[src + c] : 0.f;
            yv[k] = (in && y) ? y[src + c] : 0.f;
            lv[k] = (in && y) ? ls[c] : 0.f;
            nv[k] = (in && h_out) ? w_next[c] : 0.f;
        }
#pragma unroll
        for (int k = 0; k < N; ++k) {
            const int c = threadIdx.x + k * PN_THREADS;
            if (c >= d) continue;
            if (y) {
                xv[k] = fmaf(lv[k], yv[k], xv[k]);
                x[src + c] = xv[k];
                if (clear_y) y[src + c] = 0.f;
            }
            sum += xv[k];
        }
    } else {
        for (int c = threadIdx.x; c < d; c += PN_THREADS) {
            float v = x[src + c];
            if (y) {
                v = fmaf(ls[c], y[src + c], v);
                x[src + c] = v;
                if (clear_y) y[src + c] = 0.f;
            }
            sum += v;
        }
    }
    if (!h_out) return;
    const float mean = block_sum<PN_WAVES>(sum, scratch) / (float)d;
    float ss = 0.f;
    if (EPT > 0) {
#pragma unroll
        for (int k = 0; k < N; ++k)
            if (threadIdx.x + k * PN_THREADS < d) { const float dv = xv[k] - mean; ss = fmaf(dv, dv, ss); }
    } else {
        for (int c = threadIdx.x; c < d; c += PN_THREADS) { const float dv = x[src + c] - mean; ss = fmaf(dv, dv, ss); }
    }
    __syncthreads();                                   // (the scratch of the first sum is read by all before it is used again)
    ss = block_sum<PN_WAVES>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    if (EPT > 0) {
#pragma unroll
        for (int k = 0; k < N; ++k) {
            const int c = threadIdx.x + k * PN_THREADS;
            if (c < d) h_out[dst + c] = from_f32<T>((xv[k] - mean) * inv * nv[k]);
        }
    } else {
        for (int c = threadIdx.x; c < d; c += PN_THREADS) h_out[dst + c] = from_f32<T>((x[src + c] - mean) * inv * w_next[c]);
    }
}
}  // namespace

// x float32 [T][d] in place; y float32 [T][d] with ls float32 [d], or both null; w_next float32 [d] and h_out [n_rows][d]
// of type out_dt, or both null; rows int32 [n_rows] or null (only without y): the rows of x that are normed, in
// this order; without it n_rows = T and row i is normed into row i.
TUFF_EXPORT int tuff_scale_add_layer_norm(float* x, float* y, const float* ls, const float* w_next, float eps, void* h_out,
                                          int out_dt, const int* rows, int n_rows, int d, int clear_y, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (d <= 0 || ((y == nullptr) != (ls == nullptr)) || ((w_next == nullptr) != (h_out == nullptr)) || (rows && y)) return -2;
    dim3 grid(n_rows), block(PN_THREADS);
#define LAUNCH(E, T) hipLaunchKernelGGL((scale_add_layer_norm_kernel<T, E>), grid, block, 0, stream, x, y, ls, w_next, eps, (T*)h_out, rows, d, clear_y)
    if (d <= PN_THREADS * 4) { if (out_dt == DT_F32) LAUNCH(4, float); else LAUNCH(4, bf16_t); }
    else if (d <= PN_THREADS * 16) { if (out_dt == DT_F32) LAUNCH(16, float); else LAUNCH(16, bf16_t); }
    else { if (out_dt == DT_F32) LAUNCH(0, float); else LAUNCH(0, bf16_t); }
#undef LAUNCH
    return launch_status();
}

// x float32 [T][d] in place; y float32 [T][d] or null; w float32 [d] (with y); extra float32 [T][d] or null;
// h_out [T][d] of type out_dt or null, with w_next float32 [d] or null (no norm); y_next float32 [d] or null (with clear_y);
// y_bias float32 [d] (with y) and row_add float32 [d], each or null.
TUFF_EXPORT int tuff_post_norm_add(float* x, float* y, const float* w, float eps, float mult, const float* extra,
                                   const float* w_next, float eps_next, void* h_out, int out_dt, int n_tokens, int d,
                                   int clear_y, const float* y_next, const float* y_bias, const float* row_add, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (d <= 0 || (y && !w) || (w_next && !h_out) || (y_bias && !y)) return -2;
    dim3 grid(n_tokens), block(PN_THREADS);
    // (rows and weights lie on 16-byte borders where the row's width is a multiple of four: the caller's tensors start on them)
    const uintptr_t ends = (uintptr_t)x | (uintptr_t)y | (uintptr_t)w | (uintptr_t)extra | (uintptr_t)w_next | (uintptr_t)h_out |
                           (uintptr_t)y_next | (uintptr_t)y_bias | (uintptr_t)row_add;
    const bool vec = d % 4 == 0 && d <= PN_VEC_MAX && ends % 16 == 0;
    const int vpt = d > 1024 ? 2 : 1;
    if (vec) block = dim3(ceil_div(ceil_div(d / 4, vpt), WAVE) * WAVE);
#define LAUNCH(KERN, T) hipLaunchKernelGGL(KERN, grid, block, 0, stream, x, y, w, eps, mult, extra, w_next, eps_next, (T*)h_out, d, clear_y, y_next, y_bias, row_add)
    if (vec) {
        if (vpt == 1) {
            if (out_dt == DT_F32) LAUNCH((post_norm_add_vec_kernel<float, 1>), float); else LAUNCH((post_norm_add_vec_kernel<bf16_t, 1>), bf16_t);
        } else {
            if (out_dt == DT_F32) LAUNCH((post_norm_add_vec_kernel<float, 2>), float); else LAUNCH((post_norm_add_vec_kernel<bf16_t, 2>), bf16_t);
        }
        return launch_status();
    }
    if (d <= PN_THREADS * 8) {
        if (out_dt == DT_F32) LAUNCH((post_norm_add_regs_kernel<float, 8>), float); else LAUNCH((post_norm_add_regs_kernel<bf16_t, 8>), bf16_t);
    } else if (d <= PN_THREADS * 32) {
        if (out_dt == DT_F32) LAUNCH((post_norm_add_regs_kernel<float, 32>), float); else LAUNCH((post_norm_add_regs_kernel<bf16_t, 32>), bf16_t);
    } else {
        if (out_dt == DT_F32) LAUNCH(post_norm_add_kernel<float>, float); else LAUNCH(post_norm_add_kernel<bf16_t>, bf16_t);
    }
#undef LAUNCH
    return launch_status();
}

TUFF_EXPORT int tuff_normed_mean2(const float* a, const float* wa, const float* b, const float* wb, float eps, float coef,
                                  float* out, int n_tokens, int d, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (d <= 0) return -2;
    hipLaunchKernelGGL(normed_mean2_kernel, dim3(n_tokens), dim3(PN_THREADS), 0, stream, a, wa, b, wb, eps, coef, out, d);
    return launch_status();
}
