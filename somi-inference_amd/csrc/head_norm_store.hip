// Query, key and value norms head by head, with the keys and values into their pages.
//
// A token's row holds, as float32 sums, its query heads (dim channels each), its kv_heads key heads (dim) and its
// kv_heads value heads (vdim).  With rms(u) = sqrt(mean(u^2) + eps) over a head's channels:
//
//     q <- q / rms(q) * w_q * (1 + coef * ln(floor((p + 1) / every) + 1))          p: the token's position; coef 0: no temperature
//     k <- k / rms(k) * w_k
//     v <- v / rms(v)                                                              (norm_values; else as projected)
//
// The weights have a head's size and are shared by the heads (null: no norm of that kind).  q goes to rows of heads *
// padded channels, k to its slot of the key pages [pages, kv_heads, page, padded], v to the value pages [pages, kv_heads,
// padded, page] (transposed inside a page); channels past dim (or vdim) are written as zeros, so that kernels with one
// size for both take heads whose key and value sizes differ.  A token whose slot is negative (a padding row) stores
// nothing.  Sums, scaling and temperature are float32.  One wavefront a head.
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
head_norm_store_kernel(const float* __restrict__ rows, int64_t row_stride, const int* __restrict__ positions,
                       const int* __restrict__ slots, const float* __restrict__ wq, const float* __restrict__ wk,
                       int norm_values, float eps, float coef, int every, int heads, int kv, int dim, int vdim, int padded,
                       T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache, int page_size) {
    const int64_t t = blockIdx.x;
    const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (unit >= heads + 2 * kv) return;
    const int kind = unit < heads ? 0 : (unit < heads + kv ? 1 : 2);
    const int h = kind == 0 ? unit : (kind == 1 ? unit - heads : unit - heads - kv);
    const int slot = kind == 0 ? 0 : slots[t];
    if (slot < 0) return;
    const int size = kind == 2 ? vdim : dim;
    const float* x = rows + t * row_stride + (kind == 0 ? 0 : (int64_t)heads * dim) + (kind == 2 ? (int64_t)kv * dim : 0) +
                     (int64_t)h * size;
    const float* w = kind == 0 ? wq : (kind == 1 ? wk : nullptr);
    float ss = 0.f;
    for (int d = lane; d < size; d += 64) ss = fmaf(x[d], x[d], ss);
    ss = wave_sum(ss);
    float factor = kind == 2 ? (norm_values ? 1.0f / sqrtf(ss / (float)size + eps) : 1.0f)
                             : (w != nullptr ? 1.0f / sqrtf(ss / (float)size + eps) : 1.0f);
    if (kind == 0 && coef != 0.f) factor *= 1.0f + coef * logf((float)((positions[t] + 1) / every) + 1.0f);
    const int64_t page = slot / page_size, off = slot % page_size;
    for (int d = lane; d < padded; d += 64) {
        float v = 0.f;
        if (d < size) v = x[d] * factor * (w != nullptr ? w[d] : 1.0f);
        if (kind == 0) q_out[(t * heads + h) * padded + d] = from_float<T>(v);
        else if (kind == 1) k_cache[((page * kv + h) * page_size + off) * padded + d] = from_float<T>(v);
        else v_cache[((page * kv + h) * padded + d) * page_size + off] = from_float<T>(v);
    }
}

extern "C" int somi_head_norm_store(const float* rows, int64_t row_stride, int n_tokens, const int* positions,
                                    const int* slots, const float* wq, const float* wk, int norm_values, float eps,
                                    float coef, int every, int heads, int kv, int dim, int vdim, int padded, void* q_out,
                                    void* k_cache, void* v_cache, int page_size, int dtype, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && heads > 0 && kv > 0 && dim > 0 && vdim > 0 && page_size > 0, "head_norm_store: bad sizes");
    SOMI_REQUIRE(padded >= dim && padded >= vdim, "head_norm_store: %d channels do not hold heads of %d and %d", padded, dim, vdim);
    SOMI_REQUIRE(coef == 0.f || every > 0, "head_norm_store: a temperature that grows every %d positions", every);
    SOMI_REQUIRE(row_stride >= (int64_t)heads * dim + (int64_t)kv * (dim + vdim), "head_norm_store: rows too narrow");
    SOMI_REQUIRE(ceil_div(heads + 2 * kv, 4) <= 65535, "head_norm_store: too many heads");
    if (n_tokens == 0) return 0;
    const dim3 grid(n_tokens, ceil_div(heads + 2 * kv, 4));
#define SOMI_HNS(T)                                                                                                       \
    hipLaunchKernelGGL(head_norm_store_kernel<T>, grid, dim3(256), 0, stream, rows, row_stride, positions, slots, wq, wk, \
                       norm_values, eps, coef, every, heads, kv, dim, vdim, padded, (T*)q_out, (T*)k_cache, (T*)v_cache, \
                       page_size)
    if (dtype == SOMI_F32) SOMI_HNS(float);
    else if (dtype == SOMI_BF16) SOMI_HNS(bf16);
    else return somi_fail("head_norm_store: unknown dtype %d", dtype);
#undef SOMI_HNS
    SOMI_LAUNCH_CHECK("head_norm_store");
    return 0;
}

// A gate of one number a head on the heads' outputs: out[t, h, d] = scale * x[t, h, d] * sigmoid(g[t, h]) for d < vdim.
// x: [n, heads * padded]; g: float32, rows g_stride apart (null: no gate); out: rows of heads * vdim, out_stride apart.
template <typename T>
__global__ void __launch_bounds__(256)
head_gate_kernel(const T* __restrict__ x, const float* __restrict__ g, int64_t g_stride, float scale, int heads, int padded,
                 int vdim, T* __restrict__ out, int64_t out_stride) {
    const int64_t t = blockIdx.x;
    for (int i = blockIdx.y * 256 + threadIdx.x; i < heads * vdim; i += gridDim.y * 256) {
        const int h = i / vdim, d = i - h * vdim;
        float v = to_float(x[(t * heads + h) * padded + d]) * scale;
        if (g != nullptr) v /= 1.0f + expf(-g[t * g_stride + h]);
        out[t * out_stride + i] = from_float<T>(v);
    }
}

extern "C" int somi_head_gate(const void* x, int dtype, const float* g, int64_t g_stride, float scale, int n_tokens,
                              int heads, int padded, int vdim, void* out, int64_t out_stride, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && heads > 0 && vdim > 0 && padded >= vdim, "head_gate: bad sizes");
    SOMI_REQUIRE((g == nullptr || g_stride >= heads) && out_stride >= (int64_t)heads * vdim, "head_gate: rows too narrow");
    if (n_tokens == 0) return 0;
    const dim3 grid(n_tokens, ceil_div(heads * vdim, 1024) < 64 ? ceil_div(heads * vdim, 1024) : 64);
    if (dtype == SOMI_F32)
        hipLaunchKernelGGL(head_gate_kernel<float>, grid, dim3(256), 0, stream, (const float*)x, g, g_stride, scale, heads,
                           padded, vdim, (float*)out, out_stride);
    else if (dtype == SOMI_BF16)
        hipLaunchKernelGGL(head_gate_kernel<bf16>, grid, dim3(256), 0, stream, (const bf16*)x, g, g_stride, scale, heads,
                           padded, vdim, (bf16*)out, out_stride);
    else
        return somi_fail("head_gate: unknown dtype %d", dtype);
    SOMI_LAUNCH_CHECK("head_gate");
    return 0;
}
