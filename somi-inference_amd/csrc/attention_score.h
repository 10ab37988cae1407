// What may be done to attention scores beside scaling and a causal mask or a window, each on its own:
//
//   softcap   a scaled score s becomes softcap * tanh(s / softcap)
//   chunk     a query at position p sees only keys from chunk * floor(p / chunk) on (chunks counted from the sequence's start)
//   sink      the softmax's denominator also contains exp(sink[h]), a term without a key or a value, neither scaled nor capped
#pragma once
#include <hip/hip_runtime.h>

struct ScoreShape {
    float softcap;           // 0: none
    int chunk;               // 0: none
    const float* sink;       // [heads] float32, or null
    __host__ __device__ bool any() const { return softcap > 0.f || chunk > 0 || sink != nullptr; }
};

// What a kernel that stages keys through LDS is compiled for.
enum ScoreForm { SCORE_PLAIN = 0, SCORE_BIAS = 1, SCORE_SHAPED = 2 };

#define SCORE_LOG2E 1.44269504088896341f

// The first key that a query at position p sees.
__device__ __forceinline__ int score_first_key(int p, int window, int chunk) {
    const int lo = (window > 0 && p - window + 1 > 0) ? p - window + 1 : 0;
    if (chunk <= 0) return lo;
    const int start = p - p % chunk;
    return start > lo ? start : lo;
}

// A raw product in base-2 units, capped, less `point`: c log2(e) tanh(x / c) - point for the scaled score x = raw * unit /
// log2(e), where `unit` turns a raw product into base-2 units of an uncapped score.  tanh(y) = 1 - 2 / (exp(2 y) + 1), which is -1 and 1 at
// both ends without a clamp.
struct ScoreCap {
    float top, twice, rate;  // c log2(e), twice that, and 2 unit / c: exp(2 x / c) = exp2(raw * rate)
    float unit;
    bool on;
    __device__ ScoreCap(float softcap, float unit_) : unit(unit_), on(softcap > 0.f) {
        top = softcap * SCORE_LOG2E;
        twice = 2.f * top;
        rate = on ? 2.f * unit_ / softcap : 0.f;
    }
    // N products at once, so that the question whether there is a cap is asked once.
    template <int N, typename V> __device__ __forceinline__ void apply(V& raw, float point = 0.f) const {
        if (on) {
            const float high = top - point;
#pragma unroll
            for (int i = 0; i < N; ++i) raw[i] = fmaf(-twice, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(raw[i] * rate) + 1.0f), high);
        } else {
#pragma unroll
            for (int i = 0; i < N; ++i) raw[i] = fmaf(raw[i], unit, -point);
        }
    }
};
