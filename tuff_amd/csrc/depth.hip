// Layers whose input is a learned sum over all earlier ones, and the token shift, all in float32.
//
// tuff_depth_average, a workgroup a token:
//     x  = sum_j w[j] xs[j]            over the n streams xs [n][T][d] (the embedding and the layers' results so far);
//                                      without xs, x is read as it is
//     r  = 1 / sqrt(mean(x^2) + eps)   left in `inv` for tuff_norm_shift, or used here:
//     h  = x r w_norm                  (the next sublayer's input), or, for a step of single tokens, with the token
//     h' = h + (s - h) mix             shift: s the row the request's state holds, which then becomes h.
//
// tuff_norm_shift, for steps with portions: out[t] = h[t] + (h[t - 1] - h[t]) mix with h[t] = x[t] inv[t] w_norm formed
// again from x and the rows' inverse root mean squares (no normed row ever goes to memory and back); the row before
// a request's first token of the step is its state, which becomes the request's last row of the step.
//
// The sums over the streams run in their order and a row's sum of squares in one order that depends on d alone, and h is
// the same two products in both kernels: a token's result does not depend on how its sequence was cut into steps.
#include "common.h"
#include <math.h>

namespace {
// The shift, and the products that make h, are kept out of contraction: both kernels then give the same bits.
__device__ __forceinline__ float normed(float x, float inv, float w) {
#pragma clang fp contract(off)
    return (x * inv) * w;
}
__device__ __forceinline__ float shifted(float h, float prev, float mix) {
#pragma clang fp contract(off)
    const float step = (prev - h) * mix;
    return h + step;
}

template <int V>
__device__ __forceinline__ void load_vec(const float* p, float (&v)[V]) {
    if constexpr (V == 4) {
        const f32x4 q = *(const f32x4*)p;
        v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
    } else v[0] = p[0];
}
template <int V>
__device__ __forceinline__ void store_vec(float* p, const float (&v)[V]) {
    if constexpr (V == 4) *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]};
    else p[0] = v[0];
}
template <int V, typename T>
__device__ __forceinline__ void store_as(T* p, const float (&v)[V]) {
    if constexpr (V == 4 && sizeof(T) == 2) *(bf16x4*)p = bf16x4{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
    else if constexpr (V == 4) *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]};
    else p[0] = from_f32<T>(v[0]);
}

constexpr int AHEAD = 8;                               // streams whose loads are under way at a time

// A thread owns pieces threadIdx.x, + blockDim.x, ... (EPT of them) of V neighbouring channels of the token's row.
template <typename T, int V, int EPT, int NT>
__global__ __launch_bounds__(NT) void depth_average_kernel(const float* __restrict__ xs, long long stream, int n,
                                                           const float* __restrict__ w, float* __restrict__ x,
                                                           const float* __restrict__ norm_w, float eps, float* __restrict__ inv_out,
                                                           T* __restrict__ h_out, const float* __restrict__ mix,
                                                           float* __restrict__ state, const int* __restrict__ req_of_token,
                                                           const int* __restrict__ state_slot, int d) {
    __shared__ float scratch[NT / WAVE];
    const long long row = (long long)blockIdx.x * d;
    float v[EPT][V];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < EPT; ++k) {
        const int c = (threadIdx.x + k * NT) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) v[k][e] = 0.f;
        if (c >= d) continue;
        if (!xs) load_vec<V>(x + row + c, v[k]);
        else {
            const float* p = xs + row + c;
            for (int j0 = 0; j0 < n; j0 += AHEAD) {
                float q[AHEAD][V];
#pragma unroll
                for (int a = 0; a < AHEAD; ++a)
                    if (j0 + a < n) load_vec<V>(p + (j0 + a) * stream, q[a]);
#pragma unroll
                for (int a = 0; a < AHEAD; ++a)
                    if (j0 + a < n) {
                        const float wj = w ? w[j0 + a] : 1.f;
#pragma unroll
                        for (int e = 0; e < V; ++e) v[k][e] = fmaf(wj, q[a][e], v[k][e]);
                    }
            }
            store_vec<V>(x + row + c, v[k]);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(v[k][e], v[k][e], ss);
    }
    if (!norm_w && !inv_out) return;
    ss = block_sum<NT / WAVE>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    if (inv_out) {
        if (threadIdx.x == 0) inv_out[blockIdx.x] = inv;
        return;
    }
    float* st = mix ? state + (long long)state_slot[req_of_token[blockIdx.x]] * d : nullptr;
#pragma unroll
    for (int k = 0; k < EPT; ++k) {
        const int c = (threadIdx.x + k * NT) * V;
        if (c >= d) continue;
        float nw[V], o[V];
        load_vec<V>(norm_w + c, nw);
#pragma unroll
        for (int e = 0; e < V; ++e) o[e] = normed(v[k][e], inv, nw[e]);
        if (mix) {
            float m[V], prev[V], h[V];
            load_vec<V>(mix + c, m);
            load_vec<V>(st + c, prev);
#pragma unroll
            for (int e = 0; e < V; ++e) { h[e] = o[e]; o[e] = shifted(h[e], prev[e], m[e]); }
            store_vec<V>(st + c, h);
        }
        store_as<V>(h_out + row + c, o);
    }
}

// A thread walks SHIFT_RUN neighbouring tokens of its V channels, each row being the row before for the next one.  The
// threads of a request's first token are the only ones that touch its state: they read it and then leave the request's
// last row there.
constexpr int SHIFT_RUN = 4;

template <typename T, int V>
__global__ __launch_bounds__(256) void norm_shift_kernel(const float* __restrict__ x, const float* __restrict__ inv,
                                                         const float* __restrict__ norm_w, const float* __restrict__ mix,
                                                         float* __restrict__ state, T* __restrict__ out,
                                                         const int* __restrict__ req_of_token, const int* __restrict__ q_start,
                                                         const int* __restrict__ q_len, const int* __restrict__ state_slot, int n_tokens,
                                                         int d) {
    const int t0 = blockIdx.x * SHIFT_RUN, nt = min(SHIFT_RUN, n_tokens - t0);
    const int c = (blockIdx.y * 256 + threadIdx.x) * V;
    if (c >= d) return;
    float nw[V], m[V], row[SHIFT_RUN + 1][V];             // row 0: the token before the run
    load_vec<V>(norm_w + c, nw);
    load_vec<V>(mix + c, m);
    auto normed_row = [&](int t, float (&h)[V]) {
        load_vec<V>(x + (long long)t * d + c, h);
        const float inv_t = inv[t];
#pragma unroll
        for (int e = 0; e < V; ++e) h[e] = normed(h[e], inv_t, nw[e]);
    };
    normed_row(max(t0 - 1, 0), row[0]);                   // (used only where it is the same request's)
#pragma unroll
    for (int i = 0; i < SHIFT_RUN; ++i) normed_row(t0 + min(i, nt - 1), row[i + 1]);
#pragma unroll
    for (int i = 0; i < SHIFT_RUN; ++i) {
        if (i >= nt) break;
        const int t = t0 + i, r = req_of_token[t];
        float prev[V], o[V];
#pragma unroll
        for (int e = 0; e < V; ++e) prev[e] = row[i][e];
        if (t == q_start[r]) {
            float* st = state + (long long)state_slot[r] * d + c;
            load_vec<V>(st, prev);
            float keep[V];
            normed_row(t + q_len[r] - 1, keep);
            store_vec<V>(st, keep);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) o[e] = shifted(row[i + 1][e], prev[e], m[e]);
        store_as<V>(out + (long long)t * d + c, o);
    }
}
}  // namespace

// xs float32 [n] streams of [n_tokens][d], `stream` elements apart, with w float32 [n] (null: ones), their weighted sum
// going to x float32 [n_tokens][d] (which is none of the streams); xs null: x is read and left as it is.  Then one of
//   inv_out float32 [n_tokens]: the rows' inverse root mean squares;
//   norm_w float32 [d] and h_out [n_tokens][d] of type out_dt: the normed rows, with mix float32 [d], state float32
//   [slots][d], req_of_token and state_slot (every request one token) shifted;
//   neither: the sum alone.
// d at most 16384.
TUFF_EXPORT int tuff_depth_average(const float* xs, long long stream, int n, const float* w, float* x, const float* norm_w, float eps,
                                   float* inv_out, void* h_out, int out_dt, const float* mix, float* state, const int* req_of_token,
                                   const int* state_slot, int n_tokens, int d, hipStream_t s) {
    if (n_tokens <= 0) return 0;
    if (d <= 0 || d > 16384 || (xs && n < 1) || (inv_out && norm_w) || ((norm_w == nullptr) != (h_out == nullptr)) || (mix && !h_out)) return -2;
    if (mix && (!state || !req_of_token || !state_slot)) return -2;
    if (!xs && !inv_out && !norm_w) return 0;
#define GO(T, V, EPT, NT) hipLaunchKernelGGL((depth_average_kernel<T, V, EPT, NT>), dim3(n_tokens), dim3(NT), 0, s, xs, stream, n, w, x, \
        norm_w, eps, inv_out, (T*)h_out, mix, state, req_of_token, state_slot, d)
#define SIZES(T) do { \
        if (d % 4 == 0) { \
            if (d <= 1024) GO(T, 4, 1, 256); else if (d <= 2048) GO(T, 4, 1, 512); else if (d <= 4096) GO(T, 4, 1, 1024); \
            else if (d <= 8192) GO(T, 4, 2, 1024); else GO(T, 4, 4, 1024); \
        } else { \
            if (d <= 256) GO(T, 1, 1, 256); else if (d <= 1024) GO(T, 1, 1, 1024); else if (d <= 4096) GO(T, 1, 4, 1024); \
            else GO(T, 1, 16, 1024); \
        } \
    } while (0)
    if (out_dt == DT_F32) SIZES(float); else SIZES(bf16_t);
#undef SIZES
#undef GO
    return launch_status();
}

// x float32 [n_tokens][d], inv float32 [n_tokens], norm_w and mix float32 [d], state float32 [slots][d], out [n_tokens][d] of
// type out_dt; req_of_token [n_tokens], q_start, q_len and state_slot [requests].
TUFF_EXPORT int tuff_norm_shift(const float* x, const float* inv, const float* norm_w, const float* mix, float* state, void* out, int out_dt,
                                const int* req_of_token, const int* q_start, const int* q_len, const int* state_slot, int n_tokens,
                                int d, hipStream_t s) {
    if (n_tokens <= 0) return 0;
    if (d <= 0) return -2;
    const int V = d % 4 == 0 ? 4 : 1;
    dim3 grid(ceil_div(n_tokens, SHIFT_RUN), ceil_div(d, 256 * V)), block(256);
#define GO(T, V) hipLaunchKernelGGL((norm_shift_kernel<T, V>), grid, block, 0, s, x, inv, norm_w, mix, state, (T*)out, req_of_token, \
        q_start, q_len, state_slot, n_tokens, d)
    if (out_dt == DT_F32) { if (V == 4) GO(float, 4); else GO(float, 1); }
    else { if (V == 4) GO(bf16_t, 4); else GO(bf16_t, 1); }
#undef GO
    return launch_status();
}
