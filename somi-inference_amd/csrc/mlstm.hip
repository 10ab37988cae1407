// The gates of a matrix memory with exponential gates (mLSTM), stabilised by a running maximum.
//
// Per head and token, from the two gates' projections ri and rf:
//
//     i = cap tanh((ri + b_i) / cap),     f = log sigmoid(cap tanh((rf + b_f) / cap))
//     m_t = max(f + m_(t-1), i)                                             (from 0 at a request's first token)
//     keep = exp(f + m_(t-1) - m_t),     write = exp(i - m_t),     floor = exp(-m_t)
//
// keep and write are what csrc/ssd.hip's recurrence takes, floor bounds the size of its normaliser from below.  m is kept
// in float32 in the request's state slot.  A token is the map m -> max(m + F, G) with F = f, G = i, and such maps compose
// ((F, G) then (F', G'): F + F', max(G + F', G')), so a workgroup owns one (entry, head) and scans its tokens in parallel.
// What leaves is made from the maxima as they were computed, so that the scan's rounding cancels between neighbours.
#include "common.h"

// THREADS, PER: a workgroup's threads and the neighbouring tokens of each.  SOLO: entries of a few tokens, walked one by one
// by a thread a head, THREADS heads of one entry to a workgroup.
template <int THREADS, int PER, bool SOLO>
__global__ void __launch_bounds__(THREADS)
mlstm_gates_kernel(const float* __restrict__ ri, const float* __restrict__ rf, int64_t row_stride, const float* __restrict__ bi,
                   const float* __restrict__ bf, float cap, const int* __restrict__ entry_start,
                   const int* __restrict__ state_slots, float* __restrict__ top, int heads, float* __restrict__ keep,
                   float* __restrict__ write, float* __restrict__ floor_) {
    constexpr int WAVES = THREADS / 64;
    __shared__ float wave_f[WAVES], wave_g[WAVES], last[THREADS];
    const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = SOLO ? blockIdx.y * THREADS + tid : blockIdx.y;
    if (h >= heads) return;
    const int t0 = entry_start[e], t1 = entry_start[e + 1];
    float* kept = top + (int64_t)state_slots[e] * heads + h;
    const float bias_i = bi[h], bias_f = bf[h];
    auto gates = [&](int t, float& i, float& f) {
        i = cap * tanhf((ri[(int64_t)t * row_stride + h] + bias_i) / cap);
        const float z = cap * tanhf((rf[(int64_t)t * row_stride + h] + bias_f) / cap);
        f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
    };
    auto leave = [&](int t, float i, float f, float before, float m) {
        const int64_t at = (int64_t)t * heads + h;
        keep[at] = expf(f + before - m);
        write[at] = expf(i - m);
        floor_[at] = expf(-m);
    };
    float m0 = *kept;
    if (SOLO) {
        for (int t = t0; t < t1; ++t) {
            float i, f;
            gates(t, i, f);
            const float m = fmaxf(f + m0, i);
            leave(t, i, f, m0, m);
            m0 = m;
        }
        *kept = m0;
        return;
    }
    for (int base = t0; base < t1; base += THREADS * PER) {
        float i[PER], f[PER];
        float F = 0.f, G = -INFINITY;                        // this thread's tokens as one map
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int t = base + tid * PER + j;
            i[j] = -INFINITY;                                // a token past the entry's last: the map that changes nothing
            f[j] = 0.f;
            if (t < t1) gates(t, i[j], f[j]);
            F += f[j];
            G = fmaxf(G + f[j], i[j]);
        }
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {             // the wavefront's tokens up to and with this thread's
            const float pf = __shfl_up(F, off, 64), pg = __shfl_up(G, off, 64);
            if (lane >= off) {
                G = fmaxf(pg + F, G);
                F += pf;
            }
        }
        if (lane == 63) {
            wave_f[wave] = F;
            wave_g[wave] = G;
        }
        __syncthreads();
        float m = m0;                                        // the maximum before the wavefront, then before this thread
        for (int w = 0; w < wave; ++w) m = fmaxf(m + wave_f[w], wave_g[w]);
        const float pf = __shfl_up(F, 1, 64), pg = __shfl_up(G, 1, 64);
        if (lane > 0) m = fmaxf(m + pf, pg);
        float ms[PER];
#pragma unroll
        for (int j = 0; j < PER; ++j) ms[j] = m = fmaxf(f[j] + m, i[j]);
        last[tid] = m;
        __syncthreads();
        float before = tid > 0 ? last[tid - 1] : m0;
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int t = base + tid * PER + j;
            if (t < t1) leave(t, i[j], f[j], before, ms[j]);
            before = ms[j];
        }
        m0 = last[THREADS - 1];
        __syncthreads();                                     // the reads, before the next tokens' maxima
    }
    if (tid == 0) *kept = m0;
}

// ri, rf: the gates' projections, head h of token t at t * row_stride + h; bi, bf: [heads]; top: [slots, heads], read and
// written in place; keep, write, floor_: [n_tokens, heads].  max_entry_len: the longest entry.
extern "C" int somi_mlstm_gates(const float* ri, const float* rf, int64_t row_stride, const float* bi, const float* bf, float cap,
                                const int* entry_start, const int* state_slots, float* top, int n_entries, int max_entry_len,
                                int heads, float* keep, float* write, float* floor_, hipStream_t stream) {
    SOMI_REQUIRE(n_entries >= 0 && heads > 0 && heads <= 65535 && row_stride >= heads, "mlstm_gates: bad sizes");
    SOMI_REQUIRE(cap > 0.f, "mlstm_gates: the gates' cap must be > 0, got %g", (double)cap);
    if (n_entries == 0) return 0;
#define SOMI_MLSTM(THREADS, PER, SOLO, GRID_Y)                                                                                \
    hipLaunchKernelGGL((mlstm_gates_kernel<THREADS, PER, SOLO>), dim3(n_entries, GRID_Y), dim3(THREADS), 0, stream, ri, rf,  \
                       row_stride, bi, bf, cap, entry_start, state_slots, top, heads, keep, write, floor_)
    if (max_entry_len <= 4) SOMI_MLSTM(256, 1, true, ceil_div(heads, 256));
    else if (max_entry_len <= 512) SOMI_MLSTM(256, 2, false, heads);
    else SOMI_MLSTM(1024, 2, false, heads);
#undef SOMI_MLSTM
    SOMI_LAUNCH_CHECK("mlstm_gates");
    return 0;
}
