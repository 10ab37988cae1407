// Query and key norm over a whole projection, with the keys (and the values) into their pages.
//
// A token's row holds its nq query heads, then its nkv key heads (and, unless the values are the keys, nkv value
// heads), each of D channels.  q is divided by the root mean square of ALL its nq * D values (eps inside the root)
// and multiplied by a weight of that size, in place; k likewise over its nkv * D values, and the normed k goes into
// the key pages [pages, nkv, page, D].  The value pages [pages, nkv, D, page] get the token's values: the value heads
// of the row, or, with TIED, the keys as they were projected, before the norm.  A token whose slot is negative (a
// padding row) stores nothing.  Sums and the scaling are float32.
#include "common.h"

template <typename T, bool TIED>
__global__ void __launch_bounds__(256)
qk_norm_store_kernel(T* __restrict__ rows, int64_t row_stride, const int* __restrict__ slots,
                     const float* __restrict__ wq, const float* __restrict__ wk, float eps, int nq, int nkv, int D,
                     T* __restrict__ k_cache, T* __restrict__ v_cache, int page_size) {
    __shared__ float red[16];
    const int64_t t = blockIdx.x;
    T* q = rows + t * row_stride;
    T* k = q + (int64_t)nq * D;
    const T* v = TIED ? k : k + (int64_t)nkv * D;
    const int qn = nq * D, kn = nkv * D;
    float sq = 0.f, sk = 0.f;
    for (int i = threadIdx.x; i < qn; i += 256) {
        const float x = to_float(q[i]);
        sq += x * x;
    }
    for (int i = threadIdx.x; i < kn; i += 256) {
        const float x = to_float(k[i]);
        sk += x * x;
    }
    sq = block_sum<256>(sq, red);
    sk = block_sum<256>(sk, red);
    const float iq = 1.0f / sqrtf(sq / (float)qn + eps), ik = 1.0f / sqrtf(sk / (float)kn + eps);
    for (int i = threadIdx.x; i < qn; i += 256) q[i] = from_float<T>(to_float(q[i]) * iq * wq[i]);
    const int slot = slots[t];
    if (slot < 0) return;
    const int64_t page = slot / page_size;
    const int off = slot - (int)page * page_size;
    for (int i = threadIdx.x; i < kn; i += 256) {
        const int g = i / D, d = i - g * D;
        v_cache[((page * nkv + g) * D + d) * page_size + off] = v[i];
        k_cache[((page * nkv + g) * page_size + off) * D + d] = from_float<T>(to_float(k[i]) * ik * wk[i]);
    }
}

extern "C" int somi_qk_norm_store(void* rows, int dtype, int64_t row_stride, const int* slots, const float* wq,
                                  const float* wk, float eps, int n_tokens, int nq, int nkv, int head_dim, int tied,
                                  void* k_cache, void* v_cache, int page_size, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && nq > 0 && nkv > 0 && head_dim > 0 && page_size > 0, "qk_norm_store: bad sizes");
    SOMI_REQUIRE(row_stride >= (int64_t)(nq + (tied ? 1 : 2) * nkv) * head_dim, "qk_norm_store: rows of %lld are too narrow",
                 (long long)row_stride);
    if (n_tokens == 0) return 0;
#define SOMI_QKN(T, TIED)                                                                                            \
    hipLaunchKernelGGL((qk_norm_store_kernel<T, TIED>), dim3(n_tokens), dim3(256), 0, stream, (T*)rows, row_stride, slots, \
                       wq, wk, eps, nq, nkv, head_dim, (T*)k_cache, (T*)v_cache, page_size)
    if (dtype == SOMI_F32) {
        if (tied) SOMI_QKN(float, true); else SOMI_QKN(float, false);
    } else if (dtype == SOMI_BF16) {
        if (tied) SOMI_QKN(bf16, true); else SOMI_QKN(bf16, false);
    } else {
        return somi_fail("qk_norm_store: unknown dtype %d", dtype);
    }
#undef SOMI_QKN
    SOMI_LAUNCH_CHECK("qk_norm_store");
    return 0;
}

// The same with a rotation behind the norm, key and value heads of their own sizes, and q in rows of its own: a token's row
// holds nq query heads and nkv key heads of D channels, then nkv value heads of DV.  After the two norms the first
// 2 * rot_half channels of every query and key head turn, channel j together with j + rot_half, by the angle p *
// inv_freq[j]; the rest pass.  q goes to rows of nq * padded channels, k to [pages, nkv, page, padded], v to [pages, nkv,
// padded, page]; channels past D (or DV) are zeros.  TI: the rows' type, T: the pages'.  Norms, angles and the turning are
// float32, rounded once.  A workgroup a token.
#define QKN_MAX_HALF 256

template <typename TI, typename T>
__global__ void __launch_bounds__(256)
qk_norm_rope_store_kernel(const TI* __restrict__ rows, int64_t row_stride, const int* __restrict__ positions,
                          const int* __restrict__ slots, const float* __restrict__ wq, const float* __restrict__ wk, float eps,
                          const float* __restrict__ inv_freq, int rot_half, int nq, int nkv, int D, int DV, int padded,
                          T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache, int page_size) {
    __shared__ float red[16];
    __shared__ float cs[2][QKN_MAX_HALF];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    const TI* q = rows + t * row_stride;
    const TI* k = q + (int64_t)nq * D;
    const TI* v = k + (int64_t)nkv * D;
    const int qn = nq * D, kn = nkv * D;
    const float pos = (float)positions[t];
    for (int j = tid; j < rot_half; j += 256) {
        const float angle = pos * inv_freq[j];
        cs[0][j] = cosf(angle);
        cs[1][j] = sinf(angle);
    }
    float sq = 0.f, sk = 0.f;
    for (int i = tid; i < qn; i += 256) {
        const float x = to_float(q[i]);
        sq = fmaf(x, x, sq);
    }
    for (int i = tid; i < kn; i += 256) {
        const float x = to_float(k[i]);
        sk = fmaf(x, x, sk);
    }
    sq = block_sum<256>(sq, red);
    sk = block_sum<256>(sk, red);                            // its barriers also publish cs
    const float iq = 1.0f / sqrtf(sq / (float)qn + eps), ik = 1.0f / sqrtf(sk / (float)kn + eps);
    // channel d of the head at `at`, normed and turned
    auto value = [&](const TI* x, const float* w, float inv, int at, int d) {
        if (d >= D) return 0.f;
        const float u = to_float(x[at + d]) * inv * w[at + d];
        if (d >= 2 * rot_half) return u;
        const int j = d < rot_half ? d : d - rot_half, o = d < rot_half ? d + rot_half : j;
        const float other = to_float(x[at + o]) * inv * w[at + o];
        return d < rot_half ? u * cs[0][j] - other * cs[1][j] : u * cs[0][j] + other * cs[1][j];
    };
    for (int i = tid; i < nq * padded; i += 256) {
        const int h = i / padded, d = i - h * padded;
        q_out[t * nq * padded + i] = from_float<T>(value(q, wq, iq, h * D, d));
    }
    const int slot = slots[t];
    if (slot < 0) return;
    const int64_t page = slot / page_size;
    const int off = slot - (int)page * page_size;
    for (int i = tid; i < nkv * padded; i += 256) {
        const int g = i / padded, d = i - g * padded;
        k_cache[((page * nkv + g) * page_size + off) * padded + d] = from_float<T>(value(k, wk, ik, g * D, d));
        v_cache[((page * nkv + g) * padded + d) * page_size + off] = from_float<T>(d < DV ? to_float(v[g * DV + d]) : 0.f);
    }
}

// inv_freq: [rotary_dim / 2] float32, or null for no rotation.  in_dtype: the rows'; dtype: q_out's and the pages'.
extern "C" int somi_qk_norm_rope_store(const void* rows, int in_dtype, int64_t row_stride, const int* positions, const int* slots,
                                       const float* wq, const float* wk, float eps, const float* inv_freq, int rotary_dim,
                                       int n_tokens, int nq, int nkv, int D, int DV, int padded, void* q_out, void* k_cache,
                                       void* v_cache, int page_size, int dtype, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && nq > 0 && nkv > 0 && D > 0 && DV > 0 && page_size > 0, "qk_norm_rope_store: bad sizes");
    SOMI_REQUIRE(padded >= D && padded >= DV, "qk_norm_rope_store: %d channels do not hold heads of %d and %d", padded, D, DV);
    SOMI_REQUIRE(row_stride >= (int64_t)(nq + nkv) * D + (int64_t)nkv * DV, "qk_norm_rope_store: rows of %lld are too narrow", (long long)row_stride);
    SOMI_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= D && rotary_dim / 2 <= QKN_MAX_HALF,
                 "qk_norm_rope_store: a rotation of %d channels of heads of %d", rotary_dim, D);
    if (n_tokens == 0) return 0;
    const int rot_half = inv_freq ? rotary_dim / 2 : 0;
#define SOMI_QKR(TI, T)                                                                                                    \
    hipLaunchKernelGGL((qk_norm_rope_store_kernel<TI, T>), dim3(n_tokens), dim3(256), 0, stream, (const TI*)rows, row_stride, \
                       positions, slots, wq, wk, eps, inv_freq, rot_half, nq, nkv, D, DV, padded, (T*)q_out, (T*)k_cache,  \
                       (T*)v_cache, page_size)
    if (dtype == SOMI_F32 && in_dtype == SOMI_F32) SOMI_QKR(float, float);
    else if (dtype == SOMI_BF16 && in_dtype == SOMI_F32) SOMI_QKR(float, bf16);
    else if (dtype == SOMI_BF16 && in_dtype == SOMI_BF16) SOMI_QKR(bf16, bf16);
    else return somi_fail("qk_norm_rope_store: rows of dtype %d for pages of dtype %d", in_dtype, dtype);
#undef SOMI_QKR
    SOMI_LAUNCH_CHECK("qk_norm_rope_store");
    return 0;
}
