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

// kActForgetGate: lower + (1 - lower) sigmoid(z + bias) in full f32; kActReluGlu: rows come in pairs (gate, up) and
// y[row / 2] = relu(gate) * up (of all segments of a product or of none).
enum RmiAct : uint32_t { kActNone, kActSigmoid, kActSilu, kActGeluTanh, kActForgetGate, kActReluGlu };

// Rows [row0, row0 + n) of a product: y[token * ld + row - row0] = act(result), f32 or the model's element type.
// mul (nullptr = none): the activation's result times mul[mul_tok[token] * mul_ld + row - row0], a table of the
// model's element type with mul_rows rows, looked up by the token's id.
struct RmiRowSeg {
    void *y;
    const float *bias;   // kActSigmoid, kActForgetGate; nullptr = 0
    const float *lower;  // kActForgetGate
    const void *mul;
    const uint32_t *mul_tok;
    uint32_t mul_ld, mul_rows;
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
    const float *gate;  // rows gate_ld apart: width, or 0 for one row that all tokens share (a layer scale)
    uint32_t gate_ld;
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

// What a product reads of the f32 residual stream, n values a token:
//   v = x                                        y == nullptr
//   v = x + y / sqrt(mean(y^2) + y_eps) * y_weight   otherwise: a sublayer's result that only now joins the stream
// v goes to x_out where that is given (in a product of one token never x itself: its workgroups all read x), and
// norm(v) is the product's operand; with a second part (x2, n2 values, kNormNone only) [v ; x2], the second one from
// column k2 on.
enum RmiNorm : uint32_t { kNormNone, kNormRms, kNormLayer };
struct RmiInput {
    const float *x = nullptr;
    uint32_t n = 0;
    RmiNorm norm = kNormNone;
    const float *weight = nullptr;
    float eps = 0, y_eps = 0;
    const float *y = nullptr, *y_weight = nullptr;
    float *x_out = nullptr;
    const float *x2 = nullptr;
    uint32_t n2 = 0, k2 = 0;
};
constexpr uint32_t kInputMax = 16384;    // most values of an input: a workgroup keeps a row in registers
constexpr uint32_t kGemvAddMax = 4096;   // most with y in a product of one token

// elem_bytes 2: bf16, 4: f32
// h[i][0 .. k_pad) (rows rmi_dense_ld apart) = the operand of token rows ? rows[i] : i, zeros elsewhere; h may be
// nullptr where x_out is all that is wanted.  Here x_out may be x.
int rmi_dense_input(uint32_t elem_bytes, const RmiInput &in, const uint32_t *rows, void *h, uint32_t n_tokens, uint32_t k_pad,
                    hipStream_t st);
// x[i] = table[tok[i]] * scale (table: a dense weight), with `turns` plus the sinusoidal vector of position pos0 + i:
// sin and cos in turn, of 2 pi turns[c / 2] a position; x_also: a second copy
struct RmiEmbed {
    const void *table;
    uint32_t ld, vocab, n;
    float scale;
    const double *turns;
    float *x, *x_also;
};
int rmi_dense_embed(uint32_t elem_bytes, const RmiEmbed &e, const uint32_t *tok, uint32_t pos0, uint32_t n_tokens, hipStream_t st);
// several tokens: matrix cores; a = [n_tokens] rows of k_pad elements, rmi_dense_ld apart
int rmi_dense_gemm(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiRowSegs &segs, uint32_t n_tokens, hipStream_t st);
int rmi_dense_gemm_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            uint32_t n_tokens, hipStream_t st);
// one token: the input in front of the product is part of the launch, for as many columns as a workgroup holds; the
// second form computes two products with inputs of their own side by side
bool rmi_dense_gemv_fits(uint32_t elem_bytes, uint32_t k_pad);
int rmi_dense_gemv(uint32_t elem_bytes, const RmiDense &w, const RmiInput &in, const RmiRowSegs &segs, hipStream_t st);
int rmi_dense_gemv_pair(uint32_t elem_bytes, const RmiDense &w0, const RmiInput &in0, const RmiRowSegs &segs0, const RmiDense &w1,
                        const RmiInput &in1, const RmiRowSegs &segs1, hipStream_t st);
int rmi_dense_gemv_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            hipStream_t st);
