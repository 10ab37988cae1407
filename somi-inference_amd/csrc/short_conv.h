// The short causal convolution with SiLU of the recurrent mixers (short_conv.hip), as other files of the library call it.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#define SHORT_CONV_MAX_TAPS 9        // the state kernel keeps taps - 1 <= 8 values a channel in registers

// out[t, c] = silu(sum_j taps_w[c, j] x[t - (taps - 1) + j, c] + bias[c]) per channel over time, float32; the inputs
// before an entry's first token come from conv_state ([slots, taps - 1, C] float32, oldest first: zeros for a fresh
// request), which is advanced by the entries' tokens.  x: rows row_stride apart; bias: [C] or null; max_entry_len: the
// longest entry (0: unknown).
int somi_short_conv(const void* x, int dtype, int64_t row_stride, const float* taps_w, const float* bias, int taps,
                    float* conv_state, const int* token_entry, const int* entry_start, const int* state_slots, int n_tokens,
                    int n_entries, int max_entry_len, int C, float* out, hipStream_t stream);
