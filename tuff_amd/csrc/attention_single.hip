// Paged attention of single tokens on the gfx950 matrix cores with softmax weights that keep float32's precision:
// bfloat16 queries and cache, many query heads a kv head (latent attention: all heads on one row a position).
//
// A workgroup of four waves takes one token, one kv head, sixteen of its query heads (the columns) and one part of
// the token's keys, and walks it in blocks of 128 keys:
//  * scores: a wave takes 32 keys of the block, S^T = K Q^T (v_mfma_f32_16x16x32_bf16, rows: keys, columns: heads);
//  * the waves exchange the block's maximum per head through LDS, form p = exp(s - m) in float32, and leave p there as
//    two bfloat16 numbers, its rounding and what the rounding left;
//  * values: a wave takes a quarter of the value channels over all 128 keys, O^T = V^T P^T, once with either part of p.
// Every key and every value channel is so read once a workgroup, all of a block's loads are asked for before its first
// product, and no wave holds more than its quarter of the output.  A second kernel merges a token's parts in
// ascending order and lets a head's sink (a logit without key or value) into the denominator.
//
// With a window the parts of a token are counted from the first one its window touches, so that a launch has as many
// parts as a window can touch, whatever the context.  A window may keep the sequence's first keys (keep_first): the parts
// that hold them and lie before the window's come first.
//
// A cached key row may hold `maps` keys side by side (differential attention: two softmax maps over one kv head's values).
// H then counts maps: column c of a token meets part c % maps of the row with its hd / maps query channels, zeros stand in
// its operand for the other parts, so the row is read once for all maps.  The merge then combines a head's two maps a1, a2:
// v = a1 - lambda * a2, v / sqrt(mean(v^2) + eps) * coef.
//
// Cache layout: K [page][kv_head][offset][hd], V [page][kv_head][vd][offset]; page sizes are multiples of 16, hd and vd
// multiples of 8 up to 256.
#include "common.h"
#include <math.h>

namespace {
constexpr int WAVES = 4, NT = WAVES * WAVE;
constexpr int BLOCK = 128;                 // keys a block: 32 a wave
constexpr int PSTRIDE = BLOCK + 8;         // bfloat16 elements from a head's weights to the next one's in LDS (sixteen rows in different banks)
constexpr int XCDS = 8;

__device__ __forceinline__ f32x4 mfma32(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// The part of keys that a token's slot stands for: the parts of first keys that lie before its window's (lo: the window's
// first key), then the window's.
__device__ __forceinline__ int kept_parts(int lo, int keep_first, int part_keys) {
    return min((keep_first + part_keys - 1) / part_keys, lo / part_keys);
}
__device__ __forceinline__ int part_of_slot(int slot, int lo, int keep_first, int part_keys) {
    const int kept = kept_parts(lo, keep_first, part_keys);
    return slot < kept ? slot : lo / part_keys + (slot - kept);
}

// KC: 32-wide pieces of the key size; DBW: 16-wide blocks of value channels a wave.
template <int KC, int DBW>
__global__ __launch_bounds__(NT) void single_part_kernel(const bf16_t* __restrict__ q, const bf16_t* __restrict__ k_cache,
                                                         const bf16_t* __restrict__ v_cache, float* __restrict__ ws_o,
                                                         float* __restrict__ ws_ml, const int* __restrict__ block_table, int max_blocks,
                                                         const int* __restrict__ req_of_token, const int* __restrict__ positions,
                                                         int n_tokens, int H, int Hkv, int hd, int vd, int page_size, int window, float scale,
                                                         const float* __restrict__ slopes, int part_keys, int n_slots, int chunks,
                                                         int keep_first, int maps) {
    __shared__ float red[WAVES][16];
    __shared__ __attribute__((aligned(16))) bf16_t p_hi[16 * PSTRIDE], p_lo[16 * PSTRIDE];
    // workgroups that read the same keys (the chunks of heads of one part) follow each other on one XCD
    const int j = blockIdx.x / XCDS, unit = (j / chunks) * XCDS + blockIdx.x % XCDS, chunk = j % chunks;
    if (unit >= n_tokens * Hkv * n_slots) return;
    const int slot = unit % n_slots, kvh = (unit / n_slots) % Hkv, t = unit / (n_slots * Hkv);
    const int G = H / Hkv, cols = min(16, G - chunk * 16), head0 = kvh * G + chunk * 16;
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, n16 = lane % 16, g = lane / 16;
    const int pos = positions[t];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const int key_begin = part_of_slot(slot, lo, keep_first, part_keys) * part_keys;
    if (key_begin > pos) return;
    const int key_end = min(key_begin + part_keys, pos + 1);
    const int* table = block_table + (long long)req_of_token[t] * max_blocks;
    const bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};

    bf16x8 qf[KC];
    const int qd = hd / maps, q_from = ((head0 + min(n16, cols - 1)) % maps) * qd;       // the column's part of the key row
    const bf16_t* qrow = q + ((long long)t * H + head0 + min(n16, cols - 1)) * qd;
#pragma unroll
    for (int kc = 0; kc < KC; ++kc) {
        const int k = kc * 32 + g * 8 - q_from;
        qf[kc] = (n16 < cols && k >= 0 && k < qd) ? *(const bf16x8*)(qrow + k) : zero;
    }
    const float slope = slopes ? slopes[head0 + min(n16, cols - 1)] : 0.f;

    float m_run = -INFINITY, l_run = 0.f;
    f32x4 o[DBW];
#pragma unroll
    for (int db = 0; db < DBW; ++db) o[db] = f32x4{0.f, 0.f, 0.f, 0.f};

    for (int key0 = key_begin; key0 < key_end; key0 += BLOCK) {
        if (key0 + BLOCK <= lo && key0 >= keep_first) continue;       // (uniform) the window has passed the block
        // the block's eight sixteens of keys lie in a page each: lane i fetches the i-th one's page number
        int my_page = 0;
        {
            const int k = key0 + 16 * (lane % 8);
            if (k <= pos && (k + 15 >= lo || k < keep_first)) my_page = table[k / page_size];
        }
        bf16x8 kf[2][KC];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const int k16 = key0 + 32 * wave + 16 * h;
            const bool live = k16 <= pos && (k16 + 15 >= lo || k16 < keep_first);
            const long long page = __shfl(my_page, 2 * wave + h, WAVE);
            const bf16_t* row = k_cache + ((page * Hkv + kvh) * page_size + k16 % page_size + n16) * hd;
#pragma unroll
            for (int kc = 0; kc < KC; ++kc) {
                const int k = kc * 32 + g * 8;
                kf[h][kc] = (live && k < hd) ? *(const bf16x8*)(row + k) : zero;
            }
        }
        bf16x8 vf[4][DBW];                                    // keys 32 ks + 8 g .. + 7 of channel n16 of the wave's blocks
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const int k8 = key0 + 32 * ks + 8 * g;
            const bool live = k8 <= pos && (k8 + 7 >= lo || k8 < keep_first);
            const long long page = __shfl(my_page, 2 * ks + g / 2, WAVE);
            const bf16_t* at = v_cache + (page * Hkv + kvh) * (long long)vd * page_size + k8 % page_size;
#pragma unroll
            for (int db = 0; db < DBW; ++db) {
                const int ch = (wave * DBW + db) * 16 + n16;
                vf[ks][db] = (live && ch < vd) ? *(const bf16x8*)(at + (long long)ch * page_size) : zero;
            }
        }
        // ---- scores of the wave's 32 keys: lane (column n16, group g) gets keys 4 g .. 4 g + 3 of either sixteen
        float v[2][4];
        float mx = -INFINITY;
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kc = 0; kc < KC; ++kc) s = mfma32(kf[h][kc], qf[kc], s);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = key0 + 32 * wave + 16 * h + 4 * g + e;
                v[h][e] = ((key >= lo || key < keep_first) && key <= pos) ? fmaf(s[e], scale, -slope * (float)(pos - key)) : -INFINITY;
                mx = fmaxf(mx, v[h][e]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
        if (g == 0) red[wave][n16] = mx;
        __syncthreads();
        // (a live block holds a visible key, so the maximum is finite)
        const float m_new = fmaxf(m_run, fmaxf(fmaxf(red[0][n16], red[1][n16]), fmaxf(red[2][n16], red[3][n16])));
        const float corr = __expf(m_run - m_new);
        m_run = m_new;
        float sum = 0.f;
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            bf16x4 hi, rest;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float p = __expf(v[h][e] - m_new);
                sum += p;
                hi[e] = (bf16_t)p;
                rest[e] = (bf16_t)(p - (float)hi[e]);
            }
            const int at = n16 * PSTRIDE + 32 * wave + 16 * h + 4 * g;
            *(bf16x4*)(p_hi + at) = hi;
            *(bf16x4*)(p_lo + at) = rest;
        }
        l_run = fmaf(l_run, corr, sum);                       // this wave's and lane group's share
        __syncthreads();
        // ---- O^T = O^T * corr + V^T P^T over the wave's channels
#pragma unroll
        for (int db = 0; db < DBW; ++db)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[db][e] *= corr;
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const bf16x8 ph = *(const bf16x8*)(p_hi + n16 * PSTRIDE + 32 * ks + 8 * g);
            const bf16x8 pl = *(const bf16x8*)(p_lo + n16 * PSTRIDE + 32 * ks + 8 * g);
            const int over = key0 + 32 * ks + 8 * g + 7 - pos;   // of the piece's last keys so many were never written
#pragma unroll
            for (int db = 0; db < DBW; ++db) {
                bf16x8 x = vf[ks][db];
                if (over > 0) {
#pragma unroll
                    for (int i = 0; i < 8; ++i)
                        if (i >= 8 - over) x[i] = (bf16_t)0.f;
                }
                o[db] = mfma32(x, ph, o[db]);
                o[db] = mfma32(x, pl, o[db]);
            }
        }
    }

    l_run += __shfl_xor(l_run, 16, WAVE);
    l_run += __shfl_xor(l_run, 32, WAVE);
    __syncthreads();
    if (g == 0) red[wave][n16] = l_run;
    __syncthreads();
    if (n16 >= cols) return;
    const long long at = ((long long)t * H + head0 + n16) * n_slots + slot;
    if (wave == 0 && g == 0) {
        ws_ml[at * 2] = m_run;
        ws_ml[at * 2 + 1] = (red[0][n16] + red[1][n16]) + (red[2][n16] + red[3][n16]);
    }
#pragma unroll
    for (int db = 0; db < DBW; ++db) {
        const int ch = (wave * DBW + db) * 16 + 4 * g;
        if (ch < vd) *(f32x4*)(ws_o + at * vd + ch) = o[db];
    }
}

// A workgroup a (token, head): the parts' results weighted by exp(m_part - M) over their common sum.
constexpr int MAX_SLOTS = WAVE;
constexpr int MAX_PART = 1024;             // keys; a plan's parts are longer only where a context would have more than MAX_SLOTS

template <typename T>
__global__ __launch_bounds__(256) void single_merge_kernel(const float* __restrict__ ws_o, const float* __restrict__ ws_ml, T* __restrict__ out,
                                                           const int* __restrict__ positions, const float* __restrict__ sinks, int H, int vd,
                                                           int window, int part_keys, int n_slots, int keep_first) {
    const long long row = blockIdx.x;
    const int lane = threadIdx.x % WAVE, ch = threadIdx.x;
    const int pos = positions[row / H];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const int parts = min(n_slots, kept_parts(lo, keep_first, part_keys) + pos / part_keys - lo / part_keys + 1);
    float m = -INFINITY, l = 0.f;
    if (lane < parts) {
        const float2 ml = *(const float2*)(ws_ml + (row * n_slots + lane) * 2);
        m = ml.x;
        l = ml.y;
    }
    const float sink = sinks ? sinks[row % H] : -INFINITY;
    const float M = fmaxf(wave_max(m), sink);
    const float w = lane < parts ? __expf(m - M) : 0.f;
    float L = wave_sum(w * l);
    if (sinks) L += __expf(sink - M);
    const float inv = 1.0f / L;
    const float* o = ws_o + row * n_slots * vd + ch;
    float acc = 0.f;
    for (int p0 = 0; p0 < parts; p0 += 8) {
        float x[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = (p0 + u < parts && ch < vd) ? o[(long long)(p0 + u) * vd] : 0.f;
#pragma unroll
        for (int u = 0; u < 8; ++u) acc = fmaf(__shfl(w, min(p0 + u, WAVE - 1), WAVE), x[u], acc);
    }
    if (ch < vd) out[row * vd + ch] = from_f32<T>(acc * inv);
}

// A workgroup a (token, head) of differential attention: the parts of both maps merged as above, then combined and normed
// over the head's channels.
template <typename T>
__global__ __launch_bounds__(256) void single_merge_diff_kernel(const float* __restrict__ ws_o, const float* __restrict__ ws_ml, T* __restrict__ out,
                                                                const int* __restrict__ positions, int heads, int vd, int window, int part_keys,
                                                                int n_slots, int keep_first, float lambda, float eps, float coef) {
    __shared__ float scratch[4];
    const long long row = blockIdx.x;
    const int lane = threadIdx.x % WAVE, ch = threadIdx.x;
    const int pos = positions[row / heads];
    const int lo = window > 0 ? max(0, pos - window + 1) : 0;
    const int parts = min(n_slots, kept_parts(lo, keep_first, part_keys) + pos / part_keys - lo / part_keys + 1);
    float w[2], inv[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        float m = -INFINITY, l = 0.f;
        if (lane < parts) {
            const float2 ml = *(const float2*)(ws_ml + ((2 * row + i) * n_slots + lane) * 2);
            m = ml.x;
            l = ml.y;
        }
        const float M = wave_max(m);
        w[i] = lane < parts ? __expf(m - M) : 0.f;
        inv[i] = 1.0f / wave_sum(w[i] * l);
    }
    const float* o = ws_o + 2 * row * n_slots * vd + ch;
    const long long other = (long long)n_slots * vd;           // from the first map's parts to the second's
    float acc[2] = {0.f, 0.f};
    for (int p0 = 0; p0 < parts; p0 += 4) {
        float x[2][4];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int u = 0; u < 4; ++u) x[i][u] = (p0 + u < parts && ch < vd) ? o[i * other + (long long)(p0 + u) * vd] : 0.f;
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int u = 0; u < 4; ++u) acc[i] = fmaf(__shfl(w[i], min(p0 + u, WAVE - 1), WAVE), x[i][u], acc[i]);
    }
    const float v = ch < vd ? fmaf(-lambda, acc[1] * inv[1], acc[0] * inv[0]) : 0.f;
    // the row's sum of squares: the waves' butterflies, then the waves in order
    const float ss = wave_sum(v * v);
    if (lane == 0) scratch[threadIdx.x / WAVE] = ss;
    __syncthreads();
    float sum = 0.f;
    for (int i = 0; i < (int)blockDim.x / WAVE; ++i) sum += scratch[i];
    if (ch < vd) out[row * vd + ch] = from_f32<T>(v * (coef / sqrtf(sum / (float)vd + eps)));
}
}  // namespace

// Parts a token's keys can touch with parts of part_keys keys: with a window as many as the window touches at any place, and
// those of the first keys that stay.
static int slots_of(int max_ctx_len, int window, int part_keys, int keep_first) {
    const int all = ceil_div(max_ctx_len < 1 ? 1 : max_ctx_len, part_keys);
    if (window <= 0) return all;
    const long long touched = ((long long)window + part_keys - 2) / part_keys + 1 + ceil_div(keep_first, part_keys);
    return touched < all ? (int)touched : all;
}

// How a launch is cut: *part_keys (a multiple of 128) and *n_slots parts a token, for work arrays ws_o float32
// [n_tokens * H * n_slots * vd] and ws_ml float32 [n_tokens * H * n_slots * 2].  Parts of 128 keys while that leaves at most 2,048
// workgroups, longer ones (up to 1,024 keys) beyond, and at most 64 of them.
TUFF_EXPORT int tuff_attention_single_plan(int n_tokens, int H, int Hkv, int max_ctx_len, int window, int keep_first, int* part_keys, int* n_slots) {
    if (n_tokens < 1 || Hkv < 1 || H < 1 || H % Hkv || keep_first < 0 || !part_keys || !n_slots) return -2;
    const long long rows = (long long)n_tokens * Hkv * ceil_div(H / Hkv, 16);
    int pk = BLOCK;
    while (pk < MAX_PART && rows * slots_of(max_ctx_len, window, pk, keep_first) > 2048) pk += BLOCK;
    while (slots_of(max_ctx_len, window, pk, keep_first) > MAX_SLOTS) pk += BLOCK;
    *part_keys = pk;
    *n_slots = slots_of(max_ctx_len, window, pk, keep_first);
    return 0;
}

// Row i of q [n_tokens][H * hd] and out [n_tokens][H * vd] is a token at positions[i] of request req_of_token[i], which sees
// the cached keys up to itself (the last `window` of them, if positive); part_keys and n_slots from the plan for a
// max_ctx_len that bounds every position + 1.  sinks, slopes: float32 [H] or null.  keep_first: with a window, keys before it
// are seen whatever the distance.  maps 2: a key row holds two keys of hd / 2 channels, q is [n_tokens][H][hd / 2] with a
// head's maps side by side (H counts maps, an even number a kv head), and out [n_tokens][H / 2 * vd] is what the merge makes of a
// head's two maps with lambda, eps and coef (no sinks then).
TUFF_EXPORT int tuff_attention_single(const void* q, const void* k_cache, const void* v_cache, void* out, int out_dt, float* ws_o, float* ws_ml,
                                      const int* block_table, int max_blocks, const int* req_of_token, const int* positions, int n_tokens,
                                      int H, int Hkv, int hd, int vd, int page_size, int window, float scale, const float* sinks,
                                      const float* slopes, int part_keys, int n_slots, int keep_first, int maps, float lambda, float eps,
                                      float coef, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (keep_first < 0 || maps < 1 || maps > 2 || (maps == 2 && (hd % 16 || (H / (Hkv < 1 ? 1 : Hkv)) % 2 || sinks))) return -2;
    if (window <= 0) keep_first = 0;
    if (Hkv < 1 || H < 1 || H % Hkv || hd < 8 || hd > 256 || hd % 8 || vd < 8 || vd > 256 || vd % 8 || page_size < 16 || page_size % 16) return -2;
    if (part_keys < BLOCK || part_keys % BLOCK || n_slots < 1 || n_slots > MAX_SLOTS || max_blocks < 1) return -2;
    const int chunks = ceil_div(H / Hkv, 16);
    const long long units = (long long)n_tokens * Hkv * n_slots;
    const long long groups = ceil_div_ll(units, XCDS) * XCDS * chunks;
    if (groups > 0x7fffffffll || (long long)n_tokens * H > 0x7fffffffll) return -2;
#define GO(KC, DBW) hipLaunchKernelGGL((single_part_kernel<KC, DBW>), dim3((unsigned)groups), dim3(NT), 0, stream, (const bf16_t*)q, \
        (const bf16_t*)k_cache, (const bf16_t*)v_cache, ws_o, ws_ml, block_table, max_blocks, req_of_token, positions, n_tokens, H, Hkv, hd, \
        vd, page_size, window, scale, slopes, part_keys, n_slots, chunks, keep_first, maps)
    const int widest = hd > vd ? hd : vd;
    if (widest <= 64) GO(2, 1); else if (widest <= 128) GO(4, 2); else GO(8, 4);
#undef GO
    const int rc = launch_status();
    if (rc) return rc;
    const dim3 block(ceil_div(vd, WAVE) * WAVE);
    if (maps == 2) {
        const dim3 rows(n_tokens * (H / 2));
#define MERGE(T) hipLaunchKernelGGL(single_merge_diff_kernel<T>, rows, block, 0, stream, ws_o, ws_ml, (T*)out, positions, H / 2, vd, window, part_keys, \
        n_slots, keep_first, lambda, eps, coef)
        if (out_dt == DT_F32) MERGE(float); else MERGE(bf16_t);
#undef MERGE
        return launch_status();
    }
    const dim3 grid(n_tokens * H);
    if (out_dt == DT_F32) hipLaunchKernelGGL(single_merge_kernel<float>, grid, block, 0, stream, ws_o, ws_ml, (float*)out, positions, sinks, H, vd, window, part_keys, n_slots, keep_first);
    else hipLaunchKernelGGL(single_merge_kernel<bf16_t>, grid, block, 0, stream, ws_o, ws_ml, (bf16_t*)out, positions, sinks, H, vd, window, part_keys, n_slots, keep_first);
    return launch_status();
}
