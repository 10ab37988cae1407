// minGRU, a recurrence whose gate does not look at its state, element by element:
//
//     z = sigmoid(rz + b_z),   u = rx + b_x,   c = u + 1/2 for u >= 0 and sigmoid(u) for u < 0
//     S_t = (1 - z) S_(t-1) + z c;     out = scale * S_t * silu(rg)
//
// rz, rx, rg: the products of the input with W_z, W_x and W_g (float32 sums).  Everything is float32 but the result.
//
// A step of S is the map s -> a s + b with a = 1 - z, b = z c, and maps compose: a workgroup owns GRU_CH channels of one
// entry and walks its tokens SEGS * GRU_T at a time; thread (segment, channel) composes the maps of its GRU_T tokens, the
// segments' maps meet in LDS, each thread runs the state through the segments before its own and then through its tokens.
// SEGS is 1 in steps of few tokens an entry, which run 64 channels a workgroup; else 64, with 16 channels, where an entry
// that fits one segment (a decoded token beside a prompt's portion) leaves the other segments and the meeting out.
#include "common.h"

template <typename T, int GRU_CH, int SEGS, int GRU_T>
__global__ void __launch_bounds__(GRU_CH * SEGS)
min_gru_kernel(const float* __restrict__ rows, int64_t row_stride, const float* __restrict__ bz, const float* __restrict__ bx,
               const int* __restrict__ entry_start, const int* __restrict__ state_slots, float* __restrict__ state, int width,
               float scale, T* __restrict__ out, int64_t out_stride) {
    __shared__ float map_a[SEGS][GRU_CH], map_b[SEGS][GRU_CH];
    const int e = blockIdx.x, ch = threadIdx.x % GRU_CH, seg = threadIdx.x / GRU_CH;
    const int c = blockIdx.y * GRU_CH + ch;
    const bool live = c < width;
    const int cc = live ? c : width - 1;
    const int t0 = entry_start[e], t1 = entry_start[e + 1];
    const bool alone = SEGS == 1 || t1 - t0 <= GRU_T;             // the same for the whole workgroup
    if (alone && seg > 0) return;
    float* kept = state + (int64_t)state_slots[e] * width + cc;
    float s = *kept;
    const float wz = bz[cc], wx = bx[cc];
    for (int base = t0; base < t1; base += SEGS * GRU_T) {
        const int first = base + seg * GRU_T;
        float a[GRU_T], b[GRU_T], gate[GRU_T];
#pragma unroll
        for (int i = 0; i < GRU_T; ++i) {
            const float* row = rows + (int64_t)min(first + i, t1 - 1) * row_stride + cc;
            a[i] = row[0];
            b[i] = row[width];
            gate[i] = row[2 * width];
        }
        float ca = 1.f, cb = 0.f;
#pragma unroll
        for (int i = 0; i < GRU_T; ++i) {
            const bool there = first + i < t1;
            const float zr = a[i] + wz, u = b[i] + wx;
            const float z = 1.0f / (1.0f + expf(-zr));
            const float cand = u >= 0.f ? u + 0.5f : 1.0f / (1.0f + expf(-u));
            a[i] = there ? 1.0f / (1.0f + expf(zr)) : 1.f;          // 1 - z without the subtraction
            b[i] = there ? z * cand : 0.f;
            ca *= a[i];
            cb = fmaf(a[i], cb, b[i]);
        }
        float mine = s;
        if (!alone) {
            __syncthreads();                     // the last round's maps are read
            map_a[seg][ch] = ca;
            map_b[seg][ch] = cb;
            __syncthreads();
            for (int x = 0; x < SEGS; ++x) {
                if (x == seg) mine = s;
                s = fmaf(map_a[x][ch], s, map_b[x][ch]);
            }
        }
#pragma unroll
        for (int i = 0; i < GRU_T; ++i) {
            mine = fmaf(a[i], mine, b[i]);
            if (live && first + i < t1)
                out[(int64_t)(first + i) * out_stride + c] = from_float<T>(scale * mine * (gate[i] / (1.0f + expf(-gate[i]))));
        }
        if (alone) s = mine;
    }
    if (live && seg == 0) *kept = s;
}

// rows: [n, 3 * width] (rz | rx | rg), row_stride apart; state: [slots, width]; out: rows of `width`, out_stride apart.
extern "C" int somi_min_gru(const float* rows, int64_t row_stride, const float* bz, const float* bx, const int* entry_start,
                            const int* state_slots, float* state, int n_entries, int max_entry_len, int width, float scale,
                            void* out, int64_t out_stride, int dtype, hipStream_t stream) {
    SOMI_REQUIRE(n_entries >= 0 && max_entry_len >= 0 && width > 0 && row_stride >= 3 * (int64_t)width && out_stride >= width,
                 "min_gru: bad sizes");
    SOMI_REQUIRE(ceil_div(width, 16) <= 65535, "min_gru: too many channels");
    if (n_entries == 0) return 0;
#define SOMI_GRU(T, CH, SEGS, TOKENS)                                                                                       \
    hipLaunchKernelGGL((min_gru_kernel<T, CH, SEGS, TOKENS>), dim3(n_entries, ceil_div(width, CH)), dim3(CH * SEGS), 0,     \
                       stream, rows, row_stride, bz, bx, entry_start, state_slots, state, width, scale, (T*)out, out_stride)
#define SOMI_GRU_BY_LENGTH(T)                              \
    do {                                                   \
        if (max_entry_len == 1) SOMI_GRU(T, 64, 1, 1);     \
        else if (max_entry_len <= 16) SOMI_GRU(T, 64, 1, 4); \
        else SOMI_GRU(T, 16, 64, 8);                       \
    } while (0)
    if (dtype == SOMI_F32) SOMI_GRU_BY_LENGTH(float);
    else if (dtype == SOMI_BF16) SOMI_GRU_BY_LENGTH(bf16);
    else return somi_fail("min_gru: unknown dtype %d", dtype);
#undef SOMI_GRU_BY_LENGTH
#undef SOMI_GRU
    SOMI_LAUNCH_CHECK("min_gru");
    return 0;
}
