// Row-wise kernels of the residual stream: embedding gather, RMSNorm, SwiGLU gate,
// casts and fills.  The residual stream is float32 in every mode; sums of squares
// are taken in float32 in a fixed order.
#include "common.h"

// ------------------------------------------------------------------ embedding
// out[t, :] = table[tokens[t], :] * scale as float32.  Reference: one row gather per token
// with no scale (src/lfm25_gpu.cu:725-741), which is scale = 1: the product with 1 is exact.
template <typename T, typename TO>
__global__ void embed_rows_kernel(const T* __restrict__ table, const int* __restrict__ tokens,
                                  TO* __restrict__ out, int d, float scale) {
    const int t = blockIdx.x;
    const long long row = tokens[t];
    const T* src = table + row * (long long)d;
    TO* dst = out + (long long)t * d;
    for (int i = threadIdx.x; i < d; i += blockDim.x) dst[i] = from_f32<TO>(to_f32(src[i]) * scale);
}

// out_dt: float32 (the residual stream), or the compute type for whoever reads the embedding itself.
TUFF_EXPORT int tuff_embed_rows(const void* table, int table_dt, const int* tokens, void* out, int out_dt,
                                int n_tokens, int d, float scale, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    dim3 grid(n_tokens), block(256);
#define LAUNCH(T, TO) hipLaunchKernelGGL((embed_rows_kernel<T, TO>), grid, block, 0, stream, (const T*)table, tokens, (TO*)out, d, scale)
    if (table_dt == DT_F32) { if (out_dt == DT_F32) LAUNCH(float, float); else LAUNCH(float, bf16_t); }
    else { if (out_dt == DT_F32) LAUNCH(bf16_t, float); else LAUNCH(bf16_t, bf16_t); }
#undef LAUNCH
    return launch_status();
}

// ----------------------------------------------------------------------- bias
// y[r, c] += bias[c], the sum in float32: for projections with a bias, after their product (the
// products' epilogues have none).
template <typename T>
__global__ void add_bias_kernel(T* __restrict__ y, const float* __restrict__ bias, long long n, int N) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) y[i] = from_f32<T>(to_f32(y[i]) + bias[i % N]);
}

TUFF_EXPORT int tuff_add_bias(void* y, int dt, const float* bias, long long rows, int N, hipStream_t stream) {
    const long long n = rows * N;
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (dt == DT_F32) hipLaunchKernelGGL(add_bias_kernel<float>, grid, block, 0, stream, (float*)y, bias, n, N);
    else hipLaunchKernelGGL(add_bias_kernel<bf16_t>, grid, block, 0, stream, (bf16_t*)y, bias, n, N);
    return launch_status();
}

// --------------------------------------------------------------- logits: scale and soft cap
// x <- x * scale, then, with cap > 0, x <- cap * tanh(x / cap).
__global__ void scale_cap_kernel(float* __restrict__ x, long long n, float scale, float cap) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    float v = x[i] * scale;
    if (cap > 0.f) v = cap * tanhf(v / cap);
    x[i] = v;
}

TUFF_EXPORT int tuff_scale_cap(float* x, long long n, float scale, float cap, hipStream_t stream) {
    if (n <= 0) return 0;
    hipLaunchKernelGGL(scale_cap_kernel, dim3((unsigned)ceil_div_ll(n, 256)), dim3(256), 0, stream, x, n, scale, cap);
    return launch_status();
}

// -------------------------------------------------------------------- RMSNorm
// y_i = x_i * (1 / sqrt(mean_j x_j^2 + eps)) * w_i   (src/lfm25_gpu.cu:235,244).
// `rows` (optional) gathers input rows: output row r is the norm of x[rows[r]]; rows of x lie ldx elements apart (they
// may be a column range of a wider row).
// Per-thread strided partial sums -> wave butterfly -> wave partials in order; which elements a
// thread takes depends on d alone (multiples of 4: four neighbours a step).
template <typename TW, typename TO, bool VEC>
__global__ __launch_bounds__(256) void rmsnorm_kernel(const float* __restrict__ x, const TW* __restrict__ w,
                                                      TO* __restrict__ out, const int* __restrict__ rows, int d, long long ldx,
                                                      float eps) {
    __shared__ float scratch[4];
    const int r = blockIdx.x;
    const long long src = rows ? rows[r] : r;
    const float* xr = x + src * ldx;
    TO* o = out + (long long)r * d;
    float ss = 0.f;
    if (VEC) {
        // d is a multiple of 4: four neighbouring elements a thread and step, 16-byte loads
        for (int i = threadIdx.x * 4; i < d; i += 1024) {
            const f32x4 v = *(const f32x4*)(xr + i);
            ss = fmaf(v[0], v[0], ss); ss = fmaf(v[1], v[1], ss); ss = fmaf(v[2], v[2], ss); ss = fmaf(v[3], v[3], ss);
        }
    } else {
        for (int i = threadIdx.x; i < d; i += 256) { const float v = xr[i]; ss += v * v; }
    }
    const float total = block_sum<4>(ss, scratch);
    const float inv = 1.0f / sqrtf(total / (float)d + eps);
    if (VEC) {
        for (int i = threadIdx.x * 4; i < d; i += 1024) {
            const f32x4 v = *(const f32x4*)(xr + i);
            TO y[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) y[e] = from_f32<TO>(v[e] * inv * to_f32(w[i + e]));
            if (sizeof(TO) == 2) *(uint2*)(o + i) = *(const uint2*)y;
            else *(uint4*)(o + i) = *(const uint4*)y;
        }
    } else {
        for (int i = threadIdx.x; i < d; i += 256) o[i] = from_f32<TO>(xr[i] * inv * to_f32(w[i]));
    }
}

TUFF_EXPORT int tuff_rmsnorm(const float* x, const void* w, int w_dt, void* out, int out_dt,
                             const int* rows, int n_rows, int d, long long ldx, float eps, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (d <= 0 || ldx < d) return -2;
    const bool vec = d % 4 == 0 && ldx % 4 == 0 && (uintptr_t)x % 16 == 0;
    dim3 grid(n_rows), block(256);
#define LAUNCH(TW, TO) do { \
        if (vec) hipLaunchKernelGGL((rmsnorm_kernel<TW, TO, true>), grid, block, 0, stream, x, (const TW*)w, (TO*)out, rows, d, ldx, eps); \
        else hipLaunchKernelGGL((rmsnorm_kernel<TW, TO, false>), grid, block, 0, stream, x, (const TW*)w, (TO*)out, rows, d, ldx, eps); \
    } while (0)
    if (w_dt == DT_F32 && out_dt == DT_F32) LAUNCH(float, float);
    else if (w_dt == DT_F32 && out_dt == DT_BF16) LAUNCH(float, bf16_t);
    else if (w_dt == DT_BF16 && out_dt == DT_F32) LAUNCH(bf16_t, float);
    else LAUNCH(bf16_t, bf16_t);
#undef LAUNCH
    return launch_status();
}

// --------------------------------------------------------------------- SwiGLU
// act[t, f] = g / (1 + exp(-g)) * u with g = gu[t, f], u = gu[t, F + f]
// (src/lfm25_gpu.cu:614-617), evaluated in float32.
template <typename T>
__global__ void swiglu_kernel(const T* __restrict__ gu, T* __restrict__ act, long long n, int F) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const long long t = i / F;
    const int f = (int)(i - t * F);
    const float g = to_f32(gu[t * 2 * F + f]);
    const float u = to_f32(gu[t * 2 * F + F + f]);
    act[i] = from_f32<T>(g / (1.0f + expf(-g)) * u);
}

TUFF_EXPORT int tuff_swiglu(const void* gu, void* act, int dt, int n_tokens, int F, hipStream_t stream) {
    const long long n = (long long)n_tokens * F;
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (dt == DT_F32) hipLaunchKernelGGL(swiglu_kernel<float>, grid, block, 0, stream, (const float*)gu, (float*)act, n, F);
    else hipLaunchKernelGGL(swiglu_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)gu, (bf16_t*)act, n, F);
    return launch_status();
}

// ----------------------------------------------------------------------- cast
template <typename TI, typename TO>
__global__ void cast_kernel(const TI* __restrict__ in, TO* __restrict__ out, long long n) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = from_f32<TO>(to_f32(in[i]));
}

// out[i] = in[i] + bias[i % N]: the float32 sums of a product get their bias and are rounded once.
template <typename TO>
__global__ void cast_bias_kernel(const float* __restrict__ in, const float* __restrict__ bias, TO* __restrict__ out, long long n, int N) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = from_f32<TO>(in[i] + bias[i % N]);
}

TUFF_EXPORT int tuff_cast_bias(const float* in, const float* bias, void* out, int out_dt, long long n, int N, hipStream_t stream) {
    if (n <= 0) return 0;
    if (N <= 0 || !bias) return -2;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (out_dt == DT_BF16) hipLaunchKernelGGL((cast_bias_kernel<bf16_t>), grid, block, 0, stream, in, bias, (bf16_t*)out, n, N);
    else hipLaunchKernelGGL((cast_bias_kernel<float>), grid, block, 0, stream, in, bias, (float*)out, n, N);
    return launch_status();
}

TUFF_EXPORT int tuff_cast(const void* in, int in_dt, void* out, int out_dt, long long n, hipStream_t stream) {
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (in_dt == DT_F32 && out_dt == DT_BF16) hipLaunchKernelGGL((cast_kernel<float, bf16_t>), grid, block, 0, stream, (const float*)in, (bf16_t*)out, n);
    else if (in_dt == DT_BF16 && out_dt == DT_F32) hipLaunchKernelGGL((cast_kernel<bf16_t, float>), grid, block, 0, stream, (const bf16_t*)in, (float*)out, n);
    else if (in_dt == DT_F32) hipLaunchKernelGGL((cast_kernel<float, float>), grid, block, 0, stream, (const float*)in, (float*)out, n);
    else hipLaunchKernelGGL((cast_kernel<bf16_t, bf16_t>), grid, block, 0, stream, (const bf16_t*)in, (bf16_t*)out, n);
    return launch_status();
}

// ----------------------------------------------------------------------- fill
// Sets n 32-bit words to `value`; used instead of a memset so that a caller may
// record it into a graph.
__global__ void fill_u32_kernel(uint32_t* __restrict__ p, uint32_t value, long long n) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = value;
}

TUFF_EXPORT int tuff_fill_u32(void* p, uint32_t value, long long n, hipStream_t stream) {
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    hipLaunchKernelGGL(fill_u32_kernel, grid, block, 0, stream, (uint32_t*)p, value, n);
    return launch_status();
}

// Clears one slot of several arrays: entry e of the table (two 64-bit words each) names an array's address and the
// 32-bit words a slot of it has.
__global__ void zero_slot_kernel(const long long* __restrict__ table, int slot) {
    uint32_t* base = (uint32_t*)table[2 * blockIdx.y];
    const long long words = table[2 * blockIdx.y + 1];
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < words) base[slot * words + i] = 0u;
}

TUFF_EXPORT int tuff_zero_slot(const long long* table, int n, long long most_words, int slot, hipStream_t stream) {
    if (n <= 0 || most_words <= 0) return 0;
    if (n > 65535 || slot < 0) return -2;
    hipLaunchKernelGGL(zero_slot_kernel, dim3((unsigned)ceil_div_ll(most_words, 256), n), dim3(256), 0, stream, table, slot);
    return launch_status();
}

// -------------------------------------------------------------------- scatter
// dst[idx[i]] = src[idx[n + i]] for i < n, bounds checked (a bad index writes nothing): token ids that
// a sampling kernel has left on the device go into the next step's token buffer without a trip
// to the host.
__global__ void scatter_i32_kernel(int* __restrict__ dst, int n_dst, const int* __restrict__ src, int n_src,
                                   const int* __restrict__ idx, int n) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const int d = idx[i], s = idx[n + i];
    if (d >= 0 && d < n_dst && s >= 0 && s < n_src) dst[d] = src[s];
}

TUFF_EXPORT int tuff_scatter_i32(int* dst, int n_dst, const int* src, int n_src, const int* idx, int n, hipStream_t stream) {
    if (n <= 0) return 0;
    hipLaunchKernelGGL(scatter_i32_kernel, dim3(ceil_div(n, 256)), dim3(256), 0, stream, dst, n_dst, src, n_src, idx, n);
    return launch_status();
}

// ----------------------------------------------------------------- dynamic tanh
// y_i = tanh(alpha x_i) w_i + b_i: a norm without statistics.  `rows` (optional) gathers input rows.
template <typename TO>
__global__ void dyt_kernel(const float* __restrict__ x, const float* __restrict__ w, const float* __restrict__ b,
                           const float* __restrict__ alpha, TO* __restrict__ out, const int* __restrict__ rows, int d) {
    const int r = blockIdx.x;
    const long long src = rows ? rows[r] : r;
    const float a = alpha[0];
    const float* xr = x + src * (long long)d;
    TO* o = out + (long long)r * d;
    for (int i = threadIdx.x; i < d; i += blockDim.x) o[i] = from_f32<TO>(fmaf(tanhf(a * xr[i]), w[i], b[i]));
}

TUFF_EXPORT int tuff_dyt(const float* x, const float* w, const float* b, const float* alpha, void* out, int out_dt,
                         const int* rows, int n_rows, int d, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    dim3 grid(n_rows), block(256);
    if (out_dt == DT_F32) hipLaunchKernelGGL(dyt_kernel<float>, grid, block, 0, stream, x, w, b, alpha, (float*)out, rows, d);
    else hipLaunchKernelGGL(dyt_kernel<bf16_t>, grid, block, 0, stream, x, w, b, alpha, (bf16_t*)out, rows, d);
    return launch_status();
}

// ------------------------------------------------------------- activations
// kind: 0 silu, 1 gelu (tanh form), 2 relu squared, 3 tanh, 4 sigmoid, 6 gelu (exact, with erf); evaluated in float32.
// (5 is the clamped gated form of glu_kernel below, 7 the form with parameters after this one.)
__device__ __forceinline__ float activation(float z, int kind) {
    switch (kind) {
        case 0: return z / (1.0f + expf(-z));
        case 1: return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
        case 2: { const float r = fmaxf(z, 0.f); return r * r; }
        case 3: return tanhf(z);
        case 6: return 0.5f * z * (1.0f + erff(z * 0.7071067811865476f));
        default: return 1.0f / (1.0f + expf(-z));
    }
}

// xIELU with a, b > 0: z > 0: a z^2 + z / 2;  z <= 0: (1/2 + b) (e^z - 1 - z) + z / 2.
__device__ __forceinline__ float xielu(float z, float a, float b) {
    if (z > 0.f) return fmaf(a * z, z, 0.5f * z);
    return fmaf(0.5f + b, expm1f(z) - z, 0.5f * z);
}

// act[t, f] = f(g) * u with g = gu[t, f], u = gu[t, F + f]: the gated product of a feed-forward whose
// gate and up rows are stacked, for any of the activations above; kind 5 is the clamped form
// g' sigmoid(alpha g') (u' + 1) with g' = min(g, limit), u' = clamp(u, -limit, limit).
template <typename TI, typename T>
__global__ void glu_kernel(const TI* __restrict__ gu, T* __restrict__ act, long long n, int F, int kind,
                           const float* __restrict__ bias, float limit, float alpha) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const long long t = i / F;
    const int f = (int)(i - t * F);
    float g = to_f32(gu[t * 2 * F + f]), u = to_f32(gu[t * 2 * F + F + f]);
    if (bias) { g += bias[f]; u += bias[F + f]; }
    if (kind == 5) {
        g = fminf(g, limit);
        u = fminf(fmaxf(u, -limit), limit);
        act[i] = from_f32<T>(g / (1.0f + expf(-alpha * g)) * (u + 1.0f));
        return;
    }
    act[i] = from_f32<T>(activation(g, kind) * u);
}

// in_dt: type of gu (float32 sums of a product may come in as they are); dt: type of act.  bias (float32 [2 F],
// or null) is added to gu first: the biases of the gate and of the up projection.
TUFF_EXPORT int tuff_glu(const void* gu, int in_dt, void* act, int dt, int n_tokens, int F, int kind, const float* bias,
                         float limit, float alpha, hipStream_t stream) {
    const long long n = (long long)n_tokens * F;
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (dt == DT_F32 && in_dt == DT_F32) hipLaunchKernelGGL((glu_kernel<float, float>), grid, block, 0, stream, (const float*)gu, (float*)act, n, F, kind, bias, limit, alpha);
    else if (in_dt == DT_F32) hipLaunchKernelGGL((glu_kernel<float, bf16_t>), grid, block, 0, stream, (const float*)gu, (bf16_t*)act, n, F, kind, bias, limit, alpha);
    else if (dt == DT_BF16) hipLaunchKernelGGL((glu_kernel<bf16_t, bf16_t>), grid, block, 0, stream, (const bf16_t*)gu, (bf16_t*)act, n, F, kind, bias, limit, alpha);
    else return -2;
    return launch_status();
}

// out[t, c] = f(in[t, c] + (col_bias ? col_bias[c] : 0)) * (row_gate ? g(row_gate[t * gate_stride]) : 1): an activation
// (after a bias per column, where given), optionally times one number a row (g: gate_kind, or -1 for the number as
// it is).  in and out may be the same memory.  kind 7: xIELU, a and b the two numbers at `params`.
template <typename TI, typename TO>
__global__ void act_rows_kernel(const TI* __restrict__ in, TO* __restrict__ out, long long n, int N, int kind,
                                const float* __restrict__ row_gate, int gate_stride, int gate_kind,
                                const float* __restrict__ col_bias, const float* __restrict__ params) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float z = to_f32(in[i]) + (col_bias ? col_bias[i % N] : 0.f);
    float v = kind == 7 ? xielu(z, params[0], params[1]) : activation(z, kind);
    if (row_gate) {
        const float g = row_gate[(i / N) * gate_stride];
        v *= gate_kind < 0 ? g : activation(g, gate_kind);
    }
    out[i] = from_f32<TO>(v);
}

// The same without a row gate, four neighbouring columns a thread (N a multiple of 4, both ends on borders of their pieces).
template <typename TI, typename TO>
__global__ void act_rows_vec_kernel(const TI* __restrict__ in, TO* __restrict__ out, long long n4, int N, int kind,
                                    const float* __restrict__ col_bias, const float* __restrict__ params) {
    const long long i = ((long long)blockIdx.x * blockDim.x + threadIdx.x) * 4;
    if (i >= n4 * 4) return;
    typedef TI in4 __attribute__((ext_vector_type(4)));
    typedef TO out4 __attribute__((ext_vector_type(4)));
    const in4 v = *(const in4*)(in + i);
    const f32x4 b = col_bias ? *(const f32x4*)(col_bias + i % N) : f32x4{0.f, 0.f, 0.f, 0.f};
    out4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const float z = to_f32((TI)v[e]) + b[e];
        o[e] = from_f32<TO>(kind == 7 ? xielu(z, params[0], params[1]) : activation(z, kind));
    }
    *(out4*)(out + i) = o;
}

TUFF_EXPORT int tuff_act_rows(const void* in, int in_dt, void* out, int out_dt, long long rows, int N, int kind,
                              const float* row_gate, int gate_stride, int gate_kind, const float* col_bias, const float* params,
                              hipStream_t stream) {
    const long long n = rows * N;
    if (n <= 0) return 0;
    if ((kind == 7) != (params != nullptr)) return -2;
    if (!row_gate && N % 4 == 0 && (uintptr_t)in % 16 == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)col_bias % 16 == 0) {
        const dim3 vgrid((unsigned)ceil_div_ll(n / 4, 256));
#define LAUNCH(TI, TO) hipLaunchKernelGGL((act_rows_vec_kernel<TI, TO>), vgrid, dim3(256), 0, stream, (const TI*)in, (TO*)out, n / 4, N, kind, col_bias, params)
        if (in_dt == DT_F32 && out_dt == DT_F32) LAUNCH(float, float);
        else if (in_dt == DT_F32) LAUNCH(float, bf16_t);
        else if (out_dt == DT_F32) LAUNCH(bf16_t, float);
        else LAUNCH(bf16_t, bf16_t);
#undef LAUNCH
        return launch_status();
    }
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
#define LAUNCH(TI, TO) hipLaunchKernelGGL((act_rows_kernel<TI, TO>), grid, block, 0, stream, (const TI*)in, (TO*)out, n, N, kind, row_gate, gate_stride, gate_kind, col_bias, params)
    if (in_dt == DT_F32 && out_dt == DT_F32) LAUNCH(float, float);
    else if (in_dt == DT_F32) LAUNCH(float, bf16_t);
    else if (out_dt == DT_F32) LAUNCH(bf16_t, float);
    else LAUNCH(bf16_t, bf16_t);
#undef LAUNCH
    return launch_status();
}

// out[t, c] = f(in[t, c]) * table[tokens[t], col0 + c] for c < N, zeros for N <= c < Np: an activation times a vector looked
// up by the token's id, rows as wide as the product that follows reads them.  VEC neighbouring columns a thread.
template <typename TT, typename TO, int VEC>
__global__ void act_lookup_kernel(const float* __restrict__ in, const TT* __restrict__ table, const int* __restrict__ tokens,
                                  TO* __restrict__ out, long long n, int N, int Np, int kind, long long table_stride, int col0) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const int per = Np / VEC;
    const long long t = i / per;
    const int c = (int)(i - t * per) * VEC;
    const TT* row = table + tokens[t] * table_stride + col0;
    typedef float in_v __attribute__((ext_vector_type(VEC)));
    typedef TT tab_v __attribute__((ext_vector_type(VEC)));
    typedef TO out_v __attribute__((ext_vector_type(VEC)));
    out_v o;
    if (c < N) {
        const in_v z = *(const in_v*)(in + t * N + c);
        const tab_v e = *(const tab_v*)(row + c);
#pragma unroll
        for (int k = 0; k < VEC; ++k) o[k] = from_f32<TO>(activation(z[k], kind) * to_f32((TT)e[k]));
    } else {
#pragma unroll
        for (int k = 0; k < VEC; ++k) o[k] = from_f32<TO>(0.f);
    }
    *(out_v*)(out + t * Np + c) = o;
}

// table [*][table_stride] of type table_dt, tokens int32 [rows] (ids the caller has checked), out [rows][Np] of type out_dt.
TUFF_EXPORT int tuff_act_lookup(const float* in, const void* table, int table_dt, const int* tokens, void* out, int out_dt, long long rows,
                                int N, int Np, int kind, long long table_stride, int col0, hipStream_t stream) {
    if (rows <= 0 || N <= 0) return 0;
    if (Np < N || col0 < 0 || col0 + N > table_stride || kind == 7 || kind == 5) return -2;
    const bool four = N % 4 == 0 && Np % 4 == 0 && col0 % 4 == 0 && table_stride % 4 == 0;
    const long long n = rows * (four ? Np / 4 : Np);
    const dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
#define LAUNCH(TT, TO) do { \
    if (four) hipLaunchKernelGGL((act_lookup_kernel<TT, TO, 4>), grid, block, 0, stream, in, (const TT*)table, tokens, (TO*)out, n, N, Np, kind, table_stride, col0); \
    else hipLaunchKernelGGL((act_lookup_kernel<TT, TO, 1>), grid, block, 0, stream, in, (const TT*)table, tokens, (TO*)out, n, N, Np, kind, table_stride, col0); } while (0)
    if (table_dt == DT_F32 && out_dt == DT_F32) LAUNCH(float, float);
    else if (table_dt == DT_F32) LAUNCH(float, bf16_t);
    else if (out_dt == DT_F32) LAUNCH(bf16_t, float);
    else LAUNCH(bf16_t, bf16_t);
#undef LAUNCH
    return launch_status();
}

// ------------------------------------------------------------------ column padding
// out[t, c] = c < N ? in[t, c] : 0 for c < Np: rows widened with zeros, for a product whose inner size
// must be a multiple of the kernels' load width.
template <typename T>
__global__ void pad_cols_kernel(const T* __restrict__ in, T* __restrict__ out, long long n, int N, int Np) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const long long t = i / Np;
    const int c = (int)(i - t * Np);
    out[i] = c < N ? in[t * N + c] : from_f32<T>(0.f);
}

TUFF_EXPORT int tuff_pad_cols(const void* in, void* out, int dt, long long rows, int N, int Np, hipStream_t stream) {
    const long long n = rows * Np;
    if (n <= 0) return 0;
    dim3 grid((unsigned)ceil_div_ll(n, 256)), block(256);
    if (dt == DT_F32) hipLaunchKernelGGL(pad_cols_kernel<float>, grid, block, 0, stream, (const float*)in, (float*)out, n, N, Np);
    else hipLaunchKernelGGL(pad_cols_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)in, (bf16_t*)out, n, N, Np);
    return launch_status();
}
