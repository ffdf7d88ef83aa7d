// The short causal convolution over time of a pass's projected rows, with the rows that the pass before left.
#ifndef RMI_DEVICE_CONV_H
#define RMI_DEVICE_CONV_H

#include <hip/hip_runtime.h>
#include <stdint.h>

struct ConvCtx {
    const float *u, *hist, *conv;
    uint32_t channels, taps;
};
// the convolved channel `c` of the pass's token t
__device__ __forceinline__ float conv_at(const ConvCtx &x, uint32_t t, uint32_t pos0, uint32_t c) {
    float y = 0.0f;
    for (uint32_t j = 0; j < x.taps; j++) {
        const uint32_t back = x.taps - 1 - j;  // position pos0 + t - back
        float s = 0.0f;
        if (t >= back)
            s = x.u[size_t(t - back) * x.channels + c];
        else if (pos0 + t >= back)
            s = x.hist[size_t(t + j) * x.channels + c];  // row t - back + (taps - 1)
        y = __builtin_fmaf(x.conv[c * x.taps + j], s, y);
    }
    return y;
}
// channel c's row of the history behind the pass: position pos0 + n_tokens - (taps - 1) + j, j = 0 .. taps - 2
__device__ __forceinline__ void conv_carry(const ConvCtx &x, float *hist_out, uint32_t n_tokens, uint32_t c) {
    for (uint32_t j = 0; j + 1 < x.taps; j++) {
        const uint32_t at = n_tokens + j;  // row `at` of history followed by the pass's rows
        hist_out[size_t(j) * x.channels + c] = at >= x.taps - 1 ? x.u[size_t(at - (x.taps - 1)) * x.channels + c]
                                                                : x.hist[size_t(at) * x.channels + c];
    }
}

#endif  // RMI_DEVICE_CONV_H
