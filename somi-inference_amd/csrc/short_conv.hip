// A short causal convolution over time per channel with SiLU, in front of a recurrence (short_conv.h says what it
// computes).  Two kernels: `conv`, a thread per (token, channel), and `state`, which leaves the inputs that the next step
// needs.  An entry of one token is advanced by `conv` itself (the thread that reads a channel's kept inputs is the only
// one that does), so a step of single tokens is one launch.  Sums and SiLU are float32.
#include "short_conv.h"
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
short_conv_kernel(const T* __restrict__ x, int64_t row_stride, const float* __restrict__ taps_w, const float* __restrict__ bias,
                  int taps, float* __restrict__ conv_state, const int* __restrict__ token_entry,
                  const int* __restrict__ entry_start, const int* __restrict__ state_slots, int C, float* __restrict__ out) {
    const int64_t t = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const int e = token_entry[t];
    const int i = (int)t - entry_start[e];
    const bool single = entry_start[e + 1] - entry_start[e] == 1;
    float* st = conv_state + (int64_t)state_slots[e] * (taps - 1) * C + c;       // kept input s at st[s * C]
    float acc = 0.f, seen[SHORT_CONV_MAX_TAPS];
#pragma unroll
    for (int d = 0; d < SHORT_CONV_MAX_TAPS; ++d) {
        if (d >= taps) break;
        const float w = taps_w[c * taps + taps - 1 - d];
        seen[d] = i - d >= 0 ? to_float(x[(t - d) * row_stride + c]) : st[(int64_t)(taps - 1 + i - d) * C];
        acc += w * seen[d];
    }
    if (bias != nullptr) acc += bias[c];
    out[t * C + c] = acc / (1.0f + expf(-acc));
    if (single) {
#pragma unroll
        for (int d = 0; d < SHORT_CONV_MAX_TAPS - 1; ++d) {
            if (d >= taps - 1) break;
            st[(int64_t)(taps - 2 - d) * C] = seen[d];
        }
    }
}

// After `conv`: the last taps - 1 inputs of every entry of more than one token, from the step's rows and, where the entry
// is shorter than that, from what the state held.  A thread reads all of a channel's values before it writes any.
template <typename T>
__global__ void __launch_bounds__(256)
short_conv_state_kernel(const T* __restrict__ x, int64_t row_stride, int taps, float* __restrict__ conv_state,
                        const int* __restrict__ entry_start, const int* __restrict__ state_slots, int C) {
    const int e = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const int start = entry_start[e], len = entry_start[e + 1] - start;
    if (len == 1) return;
    float* st = conv_state + (int64_t)state_slots[e] * (taps - 1) * C;
    float vals[SHORT_CONV_MAX_TAPS - 1];
#pragma unroll
    for (int s = 0; s < SHORT_CONV_MAX_TAPS - 1; ++s) {
        if (s >= taps - 1) break;
        const int j = len - (taps - 1) + s;          // index among the entry's tokens; negative: before the entry
        vals[s] = j >= 0 ? to_float(x[(int64_t)(start + j) * row_stride + c]) : st[(int64_t)(taps - 1 + j) * C + c];
    }
#pragma unroll
    for (int s = 0; s < SHORT_CONV_MAX_TAPS - 1; ++s) {
        if (s >= taps - 1) break;
        st[(int64_t)s * C + c] = vals[s];
    }
}

template <typename T>
static void short_conv_launch(const void* x, int64_t row_stride, const float* taps_w, const float* bias, int taps,
                              float* conv_state, const int* token_entry, const int* entry_start, const int* state_slots,
                              int n_tokens, int n_entries, int max_entry_len, int C, float* out, hipStream_t stream) {
    hipLaunchKernelGGL(short_conv_kernel<T>, dim3(n_tokens, ceil_div(C, 256)), dim3(256), 0, stream, (const T*)x, row_stride,
                       taps_w, bias, taps, conv_state, token_entry, entry_start, state_slots, C, out);
    if (taps > 1 && max_entry_len != 1)
        hipLaunchKernelGGL(short_conv_state_kernel<T>, dim3(n_entries, ceil_div(C, 256)), dim3(256), 0, stream, (const T*)x,
                           row_stride, taps, conv_state, entry_start, state_slots, C);
}

int somi_short_conv(const void* x, int dtype, int64_t row_stride, const float* taps_w, const float* bias, int taps,
                    float* conv_state, const int* token_entry, const int* entry_start, const int* state_slots, int n_tokens,
                    int n_entries, int max_entry_len, int C, float* out, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && n_entries >= 0 && max_entry_len >= 0 && C > 0 && row_stride >= C, "short_conv: bad sizes");
    SOMI_REQUIRE(taps >= 1 && taps <= SHORT_CONV_MAX_TAPS, "short_conv: %d taps, at most %d are supported", taps, SHORT_CONV_MAX_TAPS);
    SOMI_REQUIRE(ceil_div(C, 256) <= 65535, "short_conv: too many channels");
    if (n_tokens == 0) return 0;
    if (dtype == SOMI_F32)
        short_conv_launch<float>(x, row_stride, taps_w, bias, taps, conv_state, token_entry, entry_start, state_slots, n_tokens,
                                 n_entries, max_entry_len, C, out, stream);
    else if (dtype == SOMI_BF16)
        short_conv_launch<bf16>(x, row_stride, taps_w, bias, taps, conv_state, token_entry, entry_start, state_slots, n_tokens,
                                n_entries, max_entry_len, C, out, stream);
    else
        return somi_fail("short_conv: unknown dtype %d", dtype);
    SOMI_LAUNCH_CHECK("short_conv");
    return 0;
}

extern "C" int somi_conv_silu(const void* x, int dtype, int64_t row_stride, const float* taps_w, const float* bias, int taps,
                              float* conv_state, const int* token_entry, const int* entry_start, const int* state_slots,
                              int n_tokens, int n_entries, int max_entry_len, int C, float* out, hipStream_t stream) {
    return somi_short_conv(x, dtype, row_stride, taps_w, bias, taps, conv_state, token_entry, entry_start, state_slots,
                           n_tokens, n_entries, max_entry_len, C, out, stream);
}
