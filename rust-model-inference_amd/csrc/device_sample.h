// Greedy sampling on the device, shared by the decoder sessions: the largest logit of each position, the token it
// makes, and that token's embedding for the next step (src/models/qwen3.rs:172-191, greedy_token).
#ifndef RMI_DEVICE_SAMPLE_H
#define RMI_DEVICE_SAMPLE_H

#include <cmath>

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace {

// The step counter in HBM: the embedding kernel reads its token through it and the argmax kernel advances it,
// so the next token never visits the host.  The kernels in between get the position as a launch argument:
// reading it from HBM first would put one more memory round trip in front of their loads.  (Replaying a whole step as a HIP graph with the counter read everywhere was
// measured: 676 vs 678 token-steps/s, no gain, so the launches stay eager.)
struct StepParams {
    uint32_t step;      // position of the token being processed = row of the KV cache
    uint32_t n_prompt;  // steps below n_prompt - 1 read their token from the prompt
};

// greedy_token: the first strict maximum, the second largest value, and whether every logit is finite
struct Top {
    float best, second;
    uint32_t id, finite;
};
__device__ __forceinline__ Top top_merge(const Top &a, const Top &b) {
    Top r;
    const bool a_first = a.best > b.best || (a.best == b.best && a.id < b.id);
    const Top &hi = a_first ? a : b, &lo = a_first ? b : a;
    r.best = hi.best;
    r.id = hi.id;
    r.second = fmaxf(fmaxf(hi.second, lo.second), lo.best);
    r.finite = a.finite & b.finite;
    return r;
}
__device__ __forceinline__ Top top_block_reduce(Top t, Top *sm) {
    sm[threadIdx.x] = t;
    __syncthreads();
    for (uint32_t s = blockDim.x >> 1; s > 0; s >>= 1) {
        if (threadIdx.x < s) sm[threadIdx.x] = top_merge(sm[threadIdx.x], sm[threadIdx.x + s]);
        __syncthreads();
    }
    return sm[0];
}
__global__ __launch_bounds__(256) void argmax_partial_kernel(const float *__restrict__ logits, uint32_t n,
                                                             Top *__restrict__ partial) {
    __shared__ Top sm[256];
    logits += size_t(blockIdx.y) * n;  // token blockIdx.y of a launch over several: its logits, its partial results
    partial += size_t(blockIdx.y) * gridDim.x;
    Top t{-INFINITY, -INFINITY, 0xffffffffu, 1u};
    for (uint32_t i = blockIdx.x * 256 + threadIdx.x; i < n; i += gridDim.x * 256) {
        const float l = logits[i];
        if (!(fabsf(l) <= 3.4028234663852886e38f)) t.finite = 0;  // NaN or inf
        if (l > t.best) {
            t.second = t.best;
            t.best = l;
            t.id = i;
        } else if (l > t.second) {
            t.second = l;
        }
    }
    const Top r = top_block_reduce(t, sm);
    if (threadIdx.x == 0) partial[blockIdx.x] = r;
}
// Embed: what turns the next token into the row the next step starts from (called by the whole workgroup).
template <typename Embed>
__global__ __launch_bounds__(256) void argmax_final_kernel(const Top *__restrict__ partial, uint32_t n_partial,
                                                           StepParams *__restrict__ sp,
                                                           uint32_t *__restrict__ tok, uint32_t *__restrict__ step_argmax,
                                                           float *__restrict__ step_top2,
                                                           uint32_t *__restrict__ nonfinite_steps, Embed embed) {
    __shared__ Top sm[256];
    __shared__ uint32_t next_token;
    Top t{-INFINITY, -INFINITY, 0xffffffffu, 1u};
    for (uint32_t i = threadIdx.x; i < n_partial; i += 256) t = top_merge(t, partial[i]);
    const Top r = top_block_reduce(t, sm);
    if (threadIdx.x == 0) {
        const uint32_t step = sp->step, n_prompt = sp->n_prompt;
        step_argmax[step] = r.id;
        step_top2[2 * step] = r.best;
        step_top2[2 * step + 1] = r.second;
        if (!r.finite) atomicAdd(nonfinite_steps, 1u);
        if (step + 1 >= n_prompt) tok[step + 1] = r.id;  // the next step's token
        next_token = step + 1 >= n_prompt ? r.id : tok[step + 1];
        sp->step = step + 1;  // last kernel of the step: the next one sees the new position
    }
    __syncthreads();
    embed(next_token);  // the next step starts from its token's embedding
}

// argmax_final_kernel for position step0 + rows[blockIdx.x] (rows == nullptr: + blockIdx.x) of a pass over several
// positions; the workgroup of the last one also leaves the step counter and the next step's embedding as a single
// step expects them.
template <typename Embed>
__global__ __launch_bounds__(256) void argmax_final_batch_kernel(const Top *__restrict__ partial, uint32_t n_partial,
                                                                 StepParams *__restrict__ sp, uint32_t step0,
                                                                 const uint32_t *__restrict__ rows,
                                                                 uint32_t *__restrict__ tok, uint32_t *__restrict__ step_argmax,
                                                                 float *__restrict__ step_top2,
                                                                 uint32_t *__restrict__ nonfinite_steps, Embed embed) {
    __shared__ Top sm[256];
    __shared__ uint32_t next_token;
    partial += size_t(blockIdx.x) * n_partial;
    Top t{-INFINITY, -INFINITY, 0xffffffffu, 1u};
    for (uint32_t i = threadIdx.x; i < n_partial; i += 256) t = top_merge(t, partial[i]);
    const Top r = top_block_reduce(t, sm);
    const uint32_t step = step0 + (rows ? rows[blockIdx.x] : blockIdx.x);
    if (threadIdx.x == 0) {
        const uint32_t n_prompt = sp->n_prompt;
        step_argmax[step] = r.id;
        step_top2[2 * step] = r.best;
        step_top2[2 * step + 1] = r.second;
        if (!r.finite) atomicAdd(nonfinite_steps, 1u);
        if (step + 1 >= n_prompt) tok[step + 1] = r.id;  // the next step's token
        next_token = step + 1 >= n_prompt ? r.id : tok[step + 1];
    }
    if (blockIdx.x + 1 != gridDim.x) return;
    if (threadIdx.x == 0) sp->step = step + 1;
    __syncthreads();
    embed(next_token);
}

}  // namespace

#endif  // RMI_DEVICE_SAMPLE_H
