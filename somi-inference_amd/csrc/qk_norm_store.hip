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
// holds, as float32 sums, nq query heads and nkv key heads of D channels, then nkv value heads of DV.  After the two norms
// the first 2 * rot_half channels of every query and key head turn, channel j together with j + rot_half, by the angle p *
// inv_freq[j]; the rest pass.  q goes to rows of nq * padded channels, k to [pages, nkv, page, padded], v to [pages, nkv,
// padded, page]; channels past D (or DV) are zeros.  Norms, angles and the turning are float32, rounded once.
//
// A workgroup sums a token's two squares whole and writes the heads u0 .. u1 - 1 of its slice (the query heads, then the
// key/value heads): a step of a few tokens has several slices a token.  V neighbouring channels at a time (4 where the heads,
// the rotation's halves and the rows are multiples of 4).
#define QKN_MAX_HALF 256

template <typename T, int V>
__global__ void __launch_bounds__(256)
qk_norm_rope_store_kernel(const float* __restrict__ rows, int64_t row_stride, const int* __restrict__ positions,
                          const int* __restrict__ slots, const float* __restrict__ wq, const float* __restrict__ wk, float eps,
                          const float* __restrict__ inv_freq, int rot_half, int nq, int nkv, int D, int DV, int padded,
                          int slice, T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache, int page_size) {
    typedef __attribute__((ext_vector_type(V))) float vec;
    typedef __attribute__((ext_vector_type(V))) T tvec;
    __shared__ float red[8];
    __shared__ __attribute__((aligned(16))) float cs[2][QKN_MAX_HALF];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, wave = tid >> 6;
    const int u0 = blockIdx.y * slice, u1 = min(u0 + slice, nq + nkv);
    const float* q = rows + t * row_stride;
    const float* k = q + (int64_t)nq * D;
    const float* v = k + (int64_t)nkv * D;
    const int qn = nq * D, kn = nkv * D;
    float sq = 0.f, sk = 0.f;
    for (int i = tid * V; i < qn + kn; i += 256 * V) {       // q and k lie side by side
        const vec x = *reinterpret_cast<const vec*>(q + i);
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(x[e], x[e], ss);
        if (i < qn) sq += ss;
        else sk += ss;
    }
    const float pos = (float)positions[t];
    for (int j = tid; j < rot_half; j += 256) sincosf(pos * inv_freq[j], &cs[1][j], &cs[0][j]);
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) {
        red[wave] = sq;
        red[4 + wave] = sk;
    }
    __syncthreads();                                         // also publishes cs
    sq = (red[0] + red[1]) + (red[2] + red[3]);
    sk = (red[4] + red[5]) + (red[6] + red[7]);
    const float iq = 1.0f / sqrtf(sq / (float)qn + eps), ik = 1.0f / sqrtf(sk / (float)kn + eps);
    // channels d .. d + V - 1 of the head at `at`, normed and turned (a group of V lies on one side of every edge)
    auto value = [&](const float* x, const float* w, float inv, int at, int d) {
        vec u = 0.f;
        if (d >= D) return u;
        u = *reinterpret_cast<const vec*>(x + at + d) * inv * *reinterpret_cast<const vec*>(w + at + d);
        if (d >= 2 * rot_half) return u;
        const bool first = d < rot_half;
        const int j = first ? d : d - rot_half, o = at + (first ? d + rot_half : j);
        const vec other = *reinterpret_cast<const vec*>(x + o) * inv * *reinterpret_cast<const vec*>(w + o);
        const vec c = *reinterpret_cast<const vec*>(&cs[0][j]), sn = *reinterpret_cast<const vec*>(&cs[1][j]);
        return first ? u * c - other * sn : u * c + other * sn;
    };
    auto put = [&](T* to, vec u) {
        tvec o;
#pragma unroll
        for (int e = 0; e < V; ++e) o[e] = from_float<T>(u[e]);
        *reinterpret_cast<tvec*>(to) = o;
    };
    const int per = padded / V;                              // groups of a head (padded is a multiple of 16 where V is 4)
    for (int i = tid; i < (min(u1, nq) - u0) * per; i += 256) {
        const int h = u0 + i / per, d = i % per * V;
        put(q_out + (t * nq + h) * padded + d, value(q, wq, iq, h * D, d));
    }
    const int slot = slots[t];
    if (slot < 0) return;
    const int64_t page = slot / page_size;
    const int off = slot - (int)page * page_size;
    const int g0 = max(u0 - nq, 0), groups = u1 - nq - g0;
    for (int i = tid; i < groups * per; i += 256) {
        const int g = g0 + i / per, d = i % per * V;
        put(k_cache + ((page * nkv + g) * page_size + off) * padded + d, value(k, wk, ik, g * D, d));
    }
    for (int i = tid; i < groups * per; i += 256) {
        const int g = g0 + i / per, d = i % per * V;
        vec u = 0.f;
        if (d < DV) u = *reinterpret_cast<const vec*>(v + g * DV + d);
#pragma unroll
        for (int e = 0; e < V; ++e) v_cache[((page * nkv + g) * padded + d + e) * page_size + off] = from_float<T>(u[e]);
    }
}

// inv_freq: [rotary_dim / 2] float32, or null for no rotation.  dtype: q_out's and the pages'.
extern "C" int somi_qk_norm_rope_store(const float* rows, int64_t row_stride, const int* positions, const int* slots,
                                       const float* wq, const float* wk, float eps, const float* inv_freq, int rotary_dim,
                                       int n_tokens, int nq, int nkv, int D, int DV, int padded, void* q_out, void* k_cache,
                                       void* v_cache, int page_size, int dtype, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && nq > 0 && nkv > 0 && D > 0 && DV > 0 && page_size > 0, "qk_norm_rope_store: bad sizes");
    SOMI_REQUIRE(padded >= D && padded >= DV, "qk_norm_rope_store: %d channels do not hold heads of %d and %d", padded, D, DV);
    SOMI_REQUIRE(row_stride >= (int64_t)(nq + nkv) * D + (int64_t)nkv * DV, "qk_norm_rope_store: rows of %lld are too narrow", (long long)row_stride);
    SOMI_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= D && rotary_dim / 2 <= QKN_MAX_HALF,
                 "qk_norm_rope_store: a rotation of %d channels of heads of %d", rotary_dim, D);
    SOMI_REQUIRE(dtype == SOMI_F32 || dtype == SOMI_BF16, "qk_norm_rope_store: unknown dtype %d", dtype);
    if (n_tokens == 0) return 0;
    const int rot_half = inv_freq ? rotary_dim / 2 : 0;
    const bool vec = D % 4 == 0 && DV % 4 == 0 && padded % 4 == 0 && rot_half % 4 == 0 && row_stride % 4 == 0 &&
                     (uintptr_t)rows % 16 == 0 && (uintptr_t)wq % 16 == 0 && (uintptr_t)wk % 16 == 0 && (uintptr_t)q_out % 16 == 0 &&
                     (uintptr_t)k_cache % 16 == 0;
    // few tokens: slices of a few heads, so that some two workgroups a compute unit share the step's heads
    const int units = nq + nkv;
    const int slices = max(1, min(units, 2 * somi_units() / n_tokens));
    const int slice = ceil_div(units, slices);
    const dim3 grid(n_tokens, ceil_div(units, slice));
#define SOMI_QKR(T, V)                                                                                                      \
    hipLaunchKernelGGL((qk_norm_rope_store_kernel<T, V>), grid, dim3(256), 0, stream, rows, row_stride, positions, slots, wq, \
                       wk, eps, inv_freq, rot_half, nq, nkv, D, DV, padded, slice, (T*)q_out, (T*)k_cache, (T*)v_cache, page_size)
    if (dtype == SOMI_F32) {
        if (vec) SOMI_QKR(float, 4); else SOMI_QKR(float, 1);
    } else {
        if (vec) SOMI_QKR(bf16, 4); else SOMI_QKR(bf16, 1);
    }
#undef SOMI_QKR
    SOMI_LAUNCH_CHECK("qk_norm_rope_store");
    return 0;
}
