// Mixers over time that decoder sessions put together: short causal convolution with rotary positions and a value
// norm, softmax attention over a cache, and the gated linear recurrence (HGRN2).  Each takes one sequence's tokens
// pos0 .. pos0 + n_tokens - 1 and what earlier calls left in its cache or state.
#pragma once

#include "dense.h"

constexpr uint32_t kMaxHeadDim = 256;
constexpr uint32_t kMaxTaps = 16;
constexpr uint32_t kKeyBlock = 32;  // keys of a value block; caches hold a multiple of this

// Softmax attention with its short convolution, interleaved rotation, value norm and per-head output gate.
//   key cache    [kv_head][capacity][dk_pad]
//   value cache  [kv_head][capacity / 32][dv_pad][32]: within a block the keys of a value channel lie in the order
//                the matrix cores take the softmax weights (rmi_value_slot)
// dk_pad and dv_pad are multiples of 32 and 16; the padding of a key is zero, that of a value is never used.
struct RmiAttnShape {
    uint32_t heads, kv_heads, dim, vdim, dk_pad, dv_pad;
    uint32_t taps, rot_dims;
    float scale, eps;
    uint32_t capacity;
};
// One pass's pointers.  u: f32 [n_tokens][channels], channels = q heads | k heads | v heads, before the convolution;
// hist_in: the taps - 1 rows before it (row j = position pos0 - (taps - 1) + j; rows of positions below zero are
// never read); hist_out, another buffer, gets the taps - 1 rows before the next pass's first.
struct RmiAttnArgs {
    const float *u, *hist_in;
    float *hist_out;
    const float *conv;   // [channels][taps]
    const float *cos_t, *sin_t;  // [capacity][rot_dims / 2]
    void *q;             // [kv_head][n_tokens * heads / kv_heads][dk_pad], used by several-token passes
    void *k_cache, *v_cache;
    const float *gate;   // [n_tokens][heads], nullptr: none
    void *out;           // [token * out_ld + head * vdim + channel], the model's element type
    uint32_t out_ld, pos0, n_tokens;
    void *scratch;       // rmi_attn_scratch_bytes; its first kAttnCounters words zero, and left zero
};
constexpr uint32_t kAttnCounters = 4096;
size_t rmi_attn_scratch_bytes(const RmiAttnShape &s);

// Gated linear recurrence: S <- diag(f) S + (1 - f) v^T, o = S^T q per head, then an RMS norm over the head.
struct RmiRecurShape {
    uint32_t heads, dim, vdim, d_pad, v_pad;  // padded to 16
    float eps;
};
struct RmiRecurArgs {
    const float *q, *f, *v;  // [n_tokens][heads * dim], f = the forget gate; [n_tokens][heads * vdim]
    const float *state_in;   // [head][d_pad][v_pad]; not read at pos0 == 0
    float *state_out;        // another buffer
    const float *norm;       // [vdim]
    void *out;               // [token * out_ld + head * vdim + channel], the model's element type
    uint32_t out_ld, pos0, n_tokens;
    float *scratch;          // rmi_recur_scratch_floats(shape, most tokens of a pass)
};
size_t rmi_recur_scratch_floats(const RmiRecurShape &s, uint32_t max_tokens);

// several tokens: the convolution's launch, the attention's; the recurrence's three
int rmi_attn_pass(uint32_t elem_bytes, const RmiAttnShape &s, const RmiAttnArgs &a, hipStream_t st);
int rmi_recur_pass(uint32_t elem_bytes, const RmiRecurShape &s, const RmiRecurArgs &a, hipStream_t st);
// one token: either mixer may be left out (nullptr); both go into one launch
int rmi_mixers_step(uint32_t elem_bytes, const RmiAttnShape *as, const RmiAttnArgs *aa, const RmiRecurShape *rs, const RmiRecurArgs *ra,
                    hipStream_t st);
