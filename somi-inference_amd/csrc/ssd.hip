// State-space duality (Mamba-2): a recurrence whose decay is one number a head and token.
//
//     dt_t = softplus(raw_t + dt_bias_h),      a_t = exp(-exp(A_log_h) dt_t)                     (per head, float32)
//     S_t  = a_t S_(t-1) + dt_t B_t x_t^T,     y_t = S_t^T C_t + D_h x_t                         (S: N x P per head, from zero)
//
// with B and C shared by the heads of a group (head h reads group h / (heads / groups)).  Everything is float32.  The
// state of a request is kept column by column, [slots, heads, P, N], so that a column's N values lie side by side.
//
// A workgroup (four wavefronts) owns 4 * 64 / LPC columns of one (entry, head).  LPC neighbouring lanes share a column:
// lane group g of it holds the rows 4 (g + LPC i) .. + 3 for i < Q in registers (rows past N are padding that stays
// zero).  The tokens' B, C and x, their dt and decay go through LDS SSD_STAGE tokens at a time; the next tokens' values
// are asked of memory before the staged ones are worked on.  Per token a lane updates its rows and sums its share of y,
// the shares are added by data-parallel moves inside the column's lanes, always in one order; the lane group that has a
// token's number (modulo LPC) keeps its y, so that a stage's results leave in a few stores.  Every column evolves by
// itself and tokens run in order from the state that earlier steps left, so a prompt cut into portions, or decoded token
// by token, performs the same operations in the same order as the whole prompt in one step.
#include "common.h"

#define SSD_STAGE 16
#define SSD_WAVES 4

typedef __attribute__((ext_vector_type(4))) float ssd_f32x4;

template <int PATTERN> __device__ __forceinline__ float ssd_dpp(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), PATTERN, 0xF, 0xF, true));
}
// The sum over the LPC (4, 8 or 16) neighbouring lanes that share a column, left in all of them.
template <int LPC> __device__ __forceinline__ float ssd_group_sum(float v) {
    v += ssd_dpp<0xB1>(v);                          // the neighbour in the quad
    v += ssd_dpp<0x4E>(v);                          // the other pair of the quad
    if (LPC == 8) v += ssd_dpp<0x141>(v);           // the other quad of the half row (mirrored)
    if (LPC == 16) {
        v += ssd_dpp<0x124>(v);                     // the quad four lanes on in the row of 16
        v += ssd_dpp<0x128>(v);                     // the pair of quads eight lanes on
    }
    return v;
}
__device__ __forceinline__ float ssd_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// xbc: [n, heads * P + 2 * groups * N] float32, x then B then C, after the convolution; raw: the tokens' dt as
// projected, rows raw_stride apart; y: [n, heads * P] float32.
template <int LPC, int Q>
__global__ void __launch_bounds__(64 * SSD_WAVES)
ssd_scan_kernel(const float* __restrict__ xbc, const float* __restrict__ raw, int64_t raw_stride,
                const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ d_skip,
                const int* __restrict__ entry_start, const int* __restrict__ state_slots, float* __restrict__ state,
                int heads, int groups, int P, int N, float* __restrict__ y) {
    constexpr int ROWS = 4 * LPC * Q, WCOLS = 64 / LPC, COLS = SSD_WAVES * WCOLS, NT = 64 * SSD_WAVES;
    constexpr int PIECES = SSD_STAGE * ROWS / NT;            // values of B (and of C) a thread stages
    constexpr int XPIECES = (SSD_STAGE * COLS + NT - 1) / NT;
    static_assert(SSD_STAGE % LPC == 0, "a stage's tokens are dealt to the lane groups evenly");
    __shared__ __attribute__((aligned(16))) float sb[SSD_STAGE][ROWS];
    __shared__ __attribute__((aligned(16))) float sc[SSD_STAGE][ROWS];
    __shared__ float sx[SSD_STAGE][COLS];
    __shared__ float sdt[SSD_STAGE], sa[SSD_STAGE];
    const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int col0 = blockIdx.z * COLS, cidx = wave * WCOLS + lane / LPC, col = col0 + cidx, g = lane % LPC;
    const bool live = col < P;
    const int t0 = entry_start[e], t1 = entry_start[e + 1];
    if (t0 >= t1) return;
    const int C = heads * P + 2 * groups * N, group = h / (heads / groups);
    const float* xs = xbc + (int64_t)h * P + col0;
    const float* bs = xbc + (int64_t)heads * P + (int64_t)group * N;
    const float* cs = bs + (int64_t)groups * N;
    const float rate = expf(a_log[h]), bias = dt_bias[h], skip = d_skip[h];
    float* S = state + (((int64_t)state_slots[e] * heads + h) * P + (live ? col : 0)) * (int64_t)N;
    float s[Q][4];
#pragma unroll
    for (int q = 0; q < Q; ++q)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int n = 4 * (g + LPC * q) + x;
            s[q][x] = live && n < N ? S[n] : 0.f;
        }
    float nb[PIECES], nc[PIECES], nx[XPIECES], nraw = 0.f;
    // addresses are clamped into the entry's rows and the rows' channels; what they bring for padding is dropped when it
    // is staged
    auto fetch = [&](int base) {
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + NT * j;
            const int64_t row = (int64_t)min(base + i / ROWS, t1 - 1) * C + min(i % ROWS, N - 1);
            nb[j] = bs[row];
            nc[j] = cs[row];
        }
#pragma unroll
        for (int j = 0; j < XPIECES; ++j) {
            const int i = tid + NT * j;
            nx[j] = xs[(int64_t)min(base + min(i / COLS, SSD_STAGE - 1), t1 - 1) * C + min(i % COLS, P - 1 - col0)];
        }
        if (tid < SSD_STAGE) nraw = raw[(int64_t)min(base + tid, t1 - 1) * raw_stride + h];
    };
    fetch(t0);
    for (int base = t0; base < t1; base += SSD_STAGE) {
        __syncthreads();                                     // the last stage's reads
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + NT * j;
            sb[i / ROWS][i % ROWS] = i % ROWS < N ? nb[j] : 0.f;
            sc[i / ROWS][i % ROWS] = i % ROWS < N ? nc[j] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < XPIECES; ++j) {
            const int i = tid + NT * j;
            if (i < SSD_STAGE * COLS) sx[i / COLS][i % COLS] = col0 + i % COLS < P ? nx[j] : 0.f;
        }
        if (tid < SSD_STAGE) {
            // a token past the entry's last leaves the state as it is: dt 0, decay 1
            const float dt = base + tid < t1 ? ssd_softplus(nraw + bias) : 0.f;
            sdt[tid] = dt;
            sa[tid] = expf(-rate * dt);
        }
        __syncthreads();
        if (base + SSD_STAGE < t1) fetch(base + SSD_STAGE);
        float keep[SSD_STAGE / LPC];
#pragma unroll
        for (int tt = 0; tt < SSD_STAGE; ++tt) {
            const float a = sa[tt], u = sdt[tt] * sx[tt][cidx];
            float part[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < Q; ++q) {
                const ssd_f32x4 b4 = *reinterpret_cast<const ssd_f32x4*>(&sb[tt][4 * (g + LPC * q)]);
                const ssd_f32x4 c4 = *reinterpret_cast<const ssd_f32x4*>(&sc[tt][4 * (g + LPC * q)]);
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    s[q][x] = fmaf(a, s[q][x], b4[x] * u);
                    part[x] = fmaf(s[q][x], c4[x], part[x]);
                }
            }
            const float sum = ssd_group_sum<LPC>((part[0] + part[1]) + (part[2] + part[3]));
            if (g == tt % LPC) keep[tt / LPC] = sum;
        }
#pragma unroll
        for (int k = 0; k < SSD_STAGE / LPC; ++k) {
            const int tt = k * LPC + g;
            if (live && base + tt < t1) y[((int64_t)(base + tt) * heads + h) * P + col] = fmaf(skip, sx[tt][cidx], keep[k]);
        }
    }
    if (!live) return;
#pragma unroll
    for (int q = 0; q < Q; ++q)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int n = 4 * (g + LPC * q) + x;
            if (n < N) S[n] = s[q][x];
        }
}

extern "C" int somi_ssd_scan(const float* xbc, const float* raw, int64_t raw_stride, const float* dt_bias, const float* a_log,
                             const float* d_skip, const int* entry_start, const int* state_slots, float* state, int n_entries,
                             int heads, int groups, int P, int N, float* y, hipStream_t stream) {
    SOMI_REQUIRE(n_entries >= 0 && heads > 0 && groups > 0 && heads % groups == 0 && P > 0 && N > 0, "ssd_scan: bad sizes");
    SOMI_REQUIRE(N <= 512, "ssd_scan: a state of %d rows is more than the supported 512", N);
    SOMI_REQUIRE(raw_stride >= heads, "ssd_scan: rows too narrow");
    if (n_entries == 0) return 0;
    // lanes a column: from the model's sizes only, so that a request's sums have one order in every batch
    const int lpc = N <= 16 ? 4 : N <= 32 ? 8 : 16;
    const int q = ceil_div(N, 4 * lpc), cols = SSD_WAVES * 64 / lpc;
    SOMI_REQUIRE(heads <= 65535 && ceil_div(P, cols) <= 65535, "ssd_scan: too many heads or columns");
    const dim3 grid(n_entries, heads, ceil_div(P, cols));
#define SOMI_SSD(L, QQ)                                                                                                      \
    hipLaunchKernelGGL((ssd_scan_kernel<L, QQ>), grid, dim3(64 * SSD_WAVES), 0, stream, xbc, raw, raw_stride, dt_bias, a_log, \
                       d_skip, entry_start, state_slots, state, heads, groups, P, N, y)
    if (lpc == 4) SOMI_SSD(4, 1);
    else if (lpc == 8) SOMI_SSD(8, 1);
    else if (q <= 1) SOMI_SSD(16, 1);
    else if (q <= 2) SOMI_SSD(16, 2);
    else if (q <= 3) SOMI_SSD(16, 3);
    else if (q <= 4) SOMI_SSD(16, 4);
    else SOMI_SSD(16, 8);
#undef SOMI_SSD
    SOMI_LAUNCH_CHECK("ssd_scan");
    return 0;
}

// ------------------------------------------------------------------------------------------------ gate and norm
// u = y * silu(z), each of `groups` equal parts of a row divided by its own root mean square (eps inside the root), times
// w and `scale`.  A workgroup a (token, part).  y: [n, width] float32; z: float32, rows z_stride apart; out: rows of
// `width`, out_stride apart.
template <typename T>
__global__ void __launch_bounds__(256)
gated_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ z, int64_t z_stride,
                        const float* __restrict__ w, float eps, float scale, int width, int part, T* __restrict__ out,
                        int64_t out_stride) {
    __shared__ float red[16];
    const int64_t t = blockIdx.x;
    const int at = blockIdx.y * part;
    const float* yr = y + t * width + at;
    const float* zr = z + t * z_stride + at;
    constexpr int HELD = 16;                  // values a thread keeps between the sum and the scaling
    float held[HELD], ss = 0.f;
    auto value = [&](int c) {
        const float gate = zr[c];
        return yr[c] * (gate / (1.0f + expf(-gate)));
    };
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        const int c = threadIdx.x + 256 * j;
        held[j] = c < part ? value(c) : 0.f;
        ss = fmaf(held[j], held[j], ss);
    }
    for (int c = threadIdx.x + 256 * HELD; c < part; c += 256) {
        const float v = value(c);
        ss = fmaf(v, v, ss);
    }
    ss = block_sum<256>(ss, red);
    const float inv = scale / sqrtf(ss / (float)part + eps);
    T* to = out + t * out_stride + at;
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        const int c = threadIdx.x + 256 * j;
        if (c < part) to[c] = from_float<T>(held[j] * inv * w[at + c]);
    }
    for (int c = threadIdx.x + 256 * HELD; c < part; c += 256) to[c] = from_float<T>(value(c) * inv * w[at + c]);
}

extern "C" int somi_gated_group_norm(const float* y, const float* z, int64_t z_stride, const float* w, int groups, float eps,
                                     float scale, int n_tokens, int width, void* out, int64_t out_stride, int dtype,
                                     hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && width > 0 && groups > 0 && width % groups == 0, "gated_group_norm: %d values in %d parts", width, groups);
    SOMI_REQUIRE(z_stride >= width && out_stride >= width && groups <= 65535, "gated_group_norm: bad strides");
    if (n_tokens == 0) return 0;
    const dim3 grid(n_tokens, groups);
    if (dtype == SOMI_F32)
        hipLaunchKernelGGL(gated_group_norm_kernel<float>, grid, dim3(256), 0, stream, y, z, z_stride, w, eps, scale, width,
                           width / groups, (float*)out, out_stride);
    else if (dtype == SOMI_BF16)
        hipLaunchKernelGGL(gated_group_norm_kernel<bf16>, grid, dim3(256), 0, stream, y, z, z_stride, w, eps, scale, width,
                           width / groups, (bf16*)out, out_stride);
    else
        return somi_fail("gated_group_norm: unknown dtype %d", dtype);
    SOMI_LAUNCH_CHECK("gated_group_norm");
    return 0;
}
