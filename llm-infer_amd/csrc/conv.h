// A short causal convolution over time per channel, for kernels that take several consecutive tokens of a step: the
// last inputs of a channel stay in registers from token to token.
#pragma once
#include "common.h"

#define CONV_MAX_TAPS 16

// How many tokens before token t of the step its sequence has in this step (at most taps - 1 of them matter).
__device__ __forceinline__ int conv_inside(const int* tok_slot, int t, int slot, int taps) {
    int inside = 0;
    while (inside < taps - 1 && t - inside - 1 >= 0 && tok_slot[t - inside - 1] == slot) ++inside;
    return inside;
}

// Column c of float32 rows (`at`: its element of token t's row, rows `stride` apart): u[b] is the input b tokens back.  Inputs
// before the first token that the sequence brings to the step (`inside` of them lie between) come from the sequence's history
// `hist` [taps - 1, channels] (oldest first); before position 0 (token t stands at p) they are zero.
template <int TAPS>
struct ConvWindow {
    float u[TAPS];
    __device__ __forceinline__ void start(const float* at, int64_t stride, int inside, int p, const float* hist, int channels, int c) {
#pragma unroll
        for (int b = 0; b < TAPS; ++b)
            u[b] = b <= inside ? at[-b * stride] : (p - b >= 0 ? hist[(int64_t)(TAPS - 1 - (b - inside)) * channels + c] : 0.f);
    }
    __device__ __forceinline__ void next(float v) {        // the next token of the same sequence
#pragma unroll
        for (int b = TAPS - 1; b > 0; --b) u[b] = u[b - 1];
        u[0] = v;
    }
    // the history as the next token will find it (only where no other thread still reads this column's)
    __device__ __forceinline__ void keep(float* hist, int channels, int c) const {
#pragma unroll
        for (int r = 0; r < TAPS - 1; ++r) hist[(int64_t)r * channels + c] = u[TAPS - 2 - r];
    }
    __device__ __forceinline__ float sum(const float* w, float acc) const {        // w [TAPS], the last one the token's own
#pragma unroll
        for (int b = 0; b < TAPS; ++b) acc += w[TAPS - 1 - b] * u[b];
        return acc;
    }
};

// The same sum for any number of taps, one token at a time.
__device__ __forceinline__ float conv_at(const float* at, int64_t stride, int inside, int p, const float* hist, int channels, int c,
                                         const float* w, int taps, float acc) {
    for (int b = 0; b < taps; ++b) {
        float u = 0.f;
        if (b <= inside) u = at[-b * stride];
        else if (p - b >= 0) u = hist[(int64_t)(taps - 1 - (b - inside)) * channels + c];
        acc += w[(int64_t)c * taps + (taps - 1 - b)] * u;
    }
    return acc;
}
__device__ __forceinline__ void conv_keep(float v, float* hist, int channels, int c, int taps) {
    for (int r = 0; r + 2 < taps; ++r) hist[(int64_t)r * channels + c] = hist[(int64_t)(r + 1) * channels + c];
    if (taps > 1) hist[(int64_t)(taps - 2) * channels + c] = v;
}
