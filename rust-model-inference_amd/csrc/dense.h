// Dense (bf16 or f32) weights and the products on them: the launch interface that decoder sessions use.
//
// A weight is row-major, rows of k_pad elements (the sum of its column segments, each padded with zeros to
// kDenseKAlign elements) that lie rmi_dense_ld apart, as do those of an activation; its row segments are each padded
// with zero rows to kDenseRowAlign.  Both element types share every kernel: the code works on 16-byte pieces.
// Accumulation is f32; the residual stream and everything a product writes is f32 unless its segment says otherwise.
#pragma once

#include "rmi_internal.h"

typedef uint16_t rmi_bf16;  // bits

constexpr uint32_t kDenseKAlign = 256;
constexpr uint32_t kDenseRowAlign = 16;
inline uint32_t rmi_dense_pad(uint32_t n, uint32_t to) { return (n + to - 1) / to * to; }

// Elements from row to row: an odd multiple of 128 bytes.  Rows a multiple of 256 bytes apart would put the same
// columns of many rows into few of the L2's channels, and a tile reads just that.
inline uint32_t rmi_dense_ld(uint32_t k_pad, uint32_t elem_bytes) {
    return k_pad + (size_t(k_pad) * elem_bytes % 256 == 0 ? 128 / elem_bytes : 0);
}

enum RmiAct : uint32_t { kActNone, kActSigmoid, kActSilu, kActGeluTanh, kActForgetGate };

// Rows [row0, row0 + n) of a product: y[token * ld + row - row0] = act(result), f32 or the model's element type.
struct RmiRowSeg {
    void *y;
    const float *bias;   // kActSigmoid (nullptr = none), kActForgetGate
    const float *lower;  // kActForgetGate
    uint32_t row0, n, ld;
    uint16_t act;
    uint16_t out_elem;  // 1: the model's element type, 0: f32
};
constexpr uint32_t kMaxRowSegs = 12;
struct RmiRowSegs {
    RmiRowSeg s[kMaxRowSegs];
    uint32_t start[kMaxRowSegs];  // s[i].row0, and n_rows from n_segs on: rmi_row_segs_done fills it
    uint32_t n_segs;
    uint32_t n_rows;  // padded rows of the weight
};
inline void rmi_row_segs_done(RmiRowSegs *r) {
    for (uint32_t i = 0; i < kMaxRowSegs; i++) r->start[i] = i < r->n_segs ? r->s[i].row0 : r->n_rows;
}

// x[token][row] += sum over column segments i of gate_i[token][row] * scale_i * (W_i a_i)[row].  A segment's columns
// end at k_end (padded); a null gate is one.
struct RmiColSeg {
    const float *gate;  // [token][width]
    float scale;
    uint32_t k_end;
};
constexpr uint32_t kMaxColSegs = 4;
struct RmiColSegs {
    RmiColSeg s[kMaxColSegs];
    uint32_t n_segs;
};

struct RmiDense {
    void *data = nullptr;
    uint32_t n_rows = 0;  // padded
    uint32_t k_pad = 0;
    uint32_t ld = 0;  // rmi_dense_ld(k_pad)
};

// More than 64 KiB of dynamic LDS has to be asked for (a compute unit has 160 KiB; some is left for static arrays).
constexpr uint32_t kLdsAskedFor = 144 * 1024;
template <typename K>
int rmi_allow_lds(K kernel, size_t bytes) {
    if (bytes <= 64 * 1024) return RMI_HIP_OK;
    RMI_HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, kLdsAskedFor));
    return RMI_HIP_OK;
}

// elem_bytes 2: bf16, 4: f32
// h[i][0 .. k_pad) (rows rmi_dense_ld apart) = rms_norm(x[rows ? rows[i] : i]) * weight, zeros past n
int rmi_dense_norm(uint32_t elem_bytes, const float *x, const uint32_t *rows, const float *weight, float eps, void *h,
                   uint32_t n_tokens, uint32_t n, uint32_t k_pad, hipStream_t st);
// x[i] = table[tok[i]] * scale (table: a dense weight)
int rmi_dense_embed(uint32_t elem_bytes, const RmiDense &table, const uint32_t *tok, uint32_t vocab, float scale, float *x,
                    uint32_t n_tokens, uint32_t n, hipStream_t st);
// several tokens: matrix cores; a = [n_tokens] rows of k_pad elements, rmi_dense_ld apart
int rmi_dense_gemm(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiRowSegs &segs, uint32_t n_tokens, hipStream_t st);
int rmi_dense_gemm_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            uint32_t n_tokens, hipStream_t st);
// one token: the norm in front of the product is part of the launch, for as many columns as a workgroup holds
bool rmi_dense_gemv_fits(uint32_t elem_bytes, uint32_t k_pad);
int rmi_dense_norm_gemv(uint32_t elem_bytes, const RmiDense &w, const float *x, const float *weight, float eps, uint32_t n,
                        const RmiRowSegs &segs, hipStream_t st);
int rmi_dense_gemv_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            hipStream_t st);
