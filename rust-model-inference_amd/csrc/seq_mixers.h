// Mixers over time that decoder sessions put together: short causal convolution with rotary positions and a value
// norm, softmax attention over a cache, the gated linear recurrence (HGRN2) and the gated delta rule.  Each takes one
// sequence's tokens pos0 .. pos0 + n_tokens - 1 and what earlier calls left in its cache or state.
#pragma once

#include "dense.h"

constexpr uint32_t kMaxHeadDim = 256;
constexpr uint32_t kMaxTaps = 16;
constexpr uint32_t kKeyBlock = 32;  // keys of a value block; caches hold a multiple of this

// Softmax attention with its short convolution, interleaved rotation, value norm and per-head output gate; each may
// be absent (one tap of ones, rot_dims 0, v_norm false, no gate).  With a window, a position sees itself and the
// window - 1 before it; the caches then are rings that hold at least window - 1 positions more than a pass brings.
//   key cache    [kv_head][capacity][dk_pad], position p in row p % capacity
//   value cache  [kv_head][capacity / 32][dv_pad][32]: within a block the keys of a value channel lie in the order
//                the matrix cores take the softmax weights (rmi_value_slot)
// dk_pad and dv_pad are multiples of 32 and 16; the padding of a key is zero, that of a value is never used.
struct RmiAttnShape {
    uint32_t heads, kv_heads, dim, vdim, dk_pad, dv_pad;
    uint32_t taps, rot_dims;
    float scale, eps;
    uint32_t capacity;
    uint32_t window;  // 0: everything before
    bool v_norm;
};
// Rows of a cache for sequences of up to `capacity` tokens in passes of up to pass_rows.
inline uint32_t rmi_attn_rows(uint32_t window, uint32_t pass_rows, uint32_t capacity) {
    const uint64_t ring = window ? uint64_t(window) - 1 + pass_rows : capacity;
    return rmi_dense_pad(ring < capacity ? uint32_t(ring) : capacity, kKeyBlock);
}
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

// Gated delta rule.  q, k (kv_heads of dim) and v (heads of vdim) pass a short causal convolution and silu; q and k
// become unit vectors, q also over sqrt(dim).  Per head, with the key head h / (heads / kv_heads):
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with beta = sigmoid(b) and the decay g = exp(-rate softplus(a + bias)), then o over its root mean square times norm, times gate.
struct RmiDeltaShape {
    uint32_t heads, kv_heads, dim, vdim, d_pad, v_pad;  // padded to 16
    uint32_t taps;
    float eps;
};
struct RmiDeltaArgs {
    const float *u;          // [n_tokens][channels], channels = q heads | k heads | v heads, before the convolution
    const float *hist_in;    // the taps - 1 rows before it; rows of positions below zero are never read
    float *hist_out;         // another buffer: the taps - 1 rows before the next pass's first
    const float *conv;       // [channels][taps], the last tap is the token's own
    const float *b, *a;      // [n_tokens][heads]
    const float *rate, *bias;  // [heads]
    const float *gate;       // [n_tokens][heads * vdim]
    const float *norm;       // [vdim]
    const float *state_in;   // [head][d_pad][v_pad]; not read at pos0 == 0
    float *state_out;        // another buffer
    void *out;               // [token * out_ld + head * vdim + channel], the model's element type
    uint32_t out_ld, pos0, n_tokens;
    float *scratch;          // rmi_delta_scratch_floats(shape, most tokens of a pass)
};
size_t rmi_delta_scratch_floats(const RmiDeltaShape &s, uint32_t max_tokens);

// several tokens: the convolution's launch, the attention's; the recurrence's three; the delta rule's three
int rmi_attn_pass(uint32_t elem_bytes, const RmiAttnShape &s, const RmiAttnArgs &a, hipStream_t st);
int rmi_recur_pass(uint32_t elem_bytes, const RmiRecurShape &s, const RmiRecurArgs &a, hipStream_t st);
// one token: either mixer may be left out (nullptr); both go into one launch
int rmi_mixers_step(uint32_t elem_bytes, const RmiAttnShape *as, const RmiAttnArgs *aa, const RmiRecurShape *rs, const RmiRecurArgs *ra,
                    hipStream_t st);
int rmi_delta_pass(uint32_t elem_bytes, const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st);
int rmi_delta_step(uint32_t elem_bytes, const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st);
