// Device functions of the dense-weight (bf16 / f32) kernels: the element type's conversions, the 16 x 16 matrix-core
// step both types share, wave reductions, and the activations of the epilogues.
#ifndef RMI_DEVICE_DENSE_H
#define RMI_DEVICE_DENSE_H

#include "dense.h"
#include "device_common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ rmi_bf16 f32_to_bf16(float v) { return __builtin_bit_cast(rmi_bf16, static_cast<__bf16>(v)); }
__device__ __forceinline__ float bf16_to_f32(uint32_t bits16) { return __builtin_bit_cast(float, bits16 << 16); }

template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ float from_f32<float>(float v) { return v; }
template <>
__device__ __forceinline__ rmi_bf16 from_f32<rmi_bf16>(float v) { return f32_to_bf16(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(rmi_bf16 v) { return bf16_to_f32(v); }

template <typename T>
constexpr uint32_t kPieceElems = 16 / sizeof(T);  // elements of one 16-byte piece

// four values to memory, as one store where p is aligned for it
template <typename T>
__device__ __forceinline__ void store4(T *p, f32x4 v);
template <>
__device__ __forceinline__ void store4<float>(float *p, f32x4 v) { *reinterpret_cast<f32x4 *>(p) = v; }
template <>
__device__ __forceinline__ void store4<rmi_bf16>(rmi_bf16 *p, f32x4 v) {
    const u32x2 o = {uint32_t(f32_to_bf16(v[0])) | (uint32_t(f32_to_bf16(v[1])) << 16),
                     uint32_t(f32_to_bf16(v[2])) | (uint32_t(f32_to_bf16(v[3])) << 16)};
    *reinterpret_cast<u32x2 *>(p) = o;
}

// acc[16 x 16] += A[16 x k] B[k x 16], one 16-byte piece of k per lane: lane l holds row l & 15 of A and column
// l & 15 of B, group g = l >> 4 of the pieces.  bf16: 32 values of k, one instruction.  f32: 16 values of k, four
// true-f32 instructions; the j-th takes element j of every lane's piece, i.e. k = 4g + j.  The result has column
// l & 15 and rows 4g .. 4g + 3 in the four registers.
template <typename T>
__device__ __forceinline__ f32x4 mma16(u32x4 a, u32x4 b, f32x4 acc);
template <>
__device__ __forceinline__ f32x4 mma16<rmi_bf16>(u32x4 a, u32x4 b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma16_f32(f32x4 a, f32x4 b, f32x4 acc) {
#pragma unroll
    for (int j = 0; j < 4; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], acc, 0, 0, 0);
    return acc;
}
template <>
__device__ __forceinline__ f32x4 mma16<float>(u32x4 a, u32x4 b, f32x4 acc) {
    return mma16_f32(__builtin_bit_cast(f32x4, a), __builtin_bit_cast(f32x4, b), acc);
}

// acc + the products of one piece
template <typename T>
__device__ __forceinline__ float dot_piece(u32x4 a, u32x4 b, float acc);
template <>
__device__ __forceinline__ float dot_piece<rmi_bf16>(u32x4 a, u32x4 b, float acc) {
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const uint32_t x = a[j], y = b[j];  // (a bit cast straight from a vector's element reads element 0)
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, x), __builtin_bit_cast(bf16x2, y), acc, false);
    }
    return acc;
}
template <>
__device__ __forceinline__ float dot_piece<float>(u32x4 a, u32x4 b, float acc) {
    const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int j = 0; j < 4; j++) acc = __builtin_fmaf(x[j], y[j], acc);
    return acc;
}

// sum of the wave's 64 values, in every lane; all lanes active
__device__ __forceinline__ float wave_sum_f32(float v) {
    v += dpp_f32<kDppQuadXor1>(v);
    v += dpp_f32<kDppQuadXor2>(v);
    v += dpp_f32<kDppRowHalfMirror>(v);
    v += dpp_f32<kDppRowMirror>(v);
    v += dpp_f32<kDppRowBcast15, 0xa>(v);
    v += dpp_f32<kDppRowBcast31, 0xc>(v);
    return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}
// sum / largest of the four values a column of a 16 x 16 result has in lanes l, l ^ 16, l ^ 32, l ^ 48
__device__ __forceinline__ float rows_sum_f32(float v) {
    v += __shfl_xor(v, 16);
    return v + __shfl_xor(v, 32);
}
__device__ __forceinline__ float rows_max_f32(float v) {
    v = fmaxf(v, __shfl_xor(v, 16));
    return fmaxf(v, __shfl_xor(v, 32));
}

// exp: the library's where everything is f32, the hardware's exp2 where the results become bf16 operands
template <typename T>
__device__ __forceinline__ float exp_t(float z);
template <>
__device__ __forceinline__ float exp_t<float>(float z) { return expf(z); }
template <>
__device__ __forceinline__ float exp_t<rmi_bf16>(float z) { return __builtin_amdgcn_exp2f(z * 1.44269504088896340736f); }
template <typename T>
__device__ __forceinline__ float rcp_t(float z);
template <>
__device__ __forceinline__ float rcp_t<float>(float z) { return 1.0f / z; }
template <>
__device__ __forceinline__ float rcp_t<rmi_bf16>(float z) { return __builtin_amdgcn_rcpf(z); }

template <typename T>
__device__ __forceinline__ float sigmoid_t(float z) { return rcp_t<T>(1.0f + exp_t<T>(-z)); }

// log(1 + e^z) in full f32
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// What a row segment of a product does with its result z (kActReluGlu: its two rows, in the epilogues themselves).
template <typename T>
__device__ __forceinline__ float apply_act(uint32_t act, float z, float bias, float lower) {
    switch (act) {
        case kActSigmoid: return sigmoid_t<T>(z + bias);
        case kActSilu: return z * sigmoid_t<T>(z);
        case kActGeluTanh:  // z/2 (1 + tanh u) = z sigmoid(2u)
            return z * sigmoid_t<T>(1.59576912160573071176f * __builtin_fmaf(0.044715f * z * z, z, z));
        case kActForgetGate: return __builtin_fmaf(1.0f - lower, sigmoid_t<float>(z + bias), lower);
        default: return z;
    }
}

// which row segment a row lies in: the starts sit side by side (unused ones at the end of the range)
__device__ __forceinline__ uint32_t seg_of(const RmiRowSegs &rs, uint32_t row) {
    uint32_t si = 0;
#pragma unroll
    for (uint32_t i = 1; i < kMaxRowSegs; i++) si += row >= rs.start[i] ? 1u : 0u;
    return si;
}

// the row of a segment's table that token t of the pass picks (ids past the end read the last row)
template <typename T>
__device__ __forceinline__ const T *mul_row(const RmiRowSeg &s, uint32_t t) {
    const uint32_t id = s.mul_tok[t];
    return static_cast<const T *>(s.mul) + size_t(id < s.mul_rows ? id : s.mul_rows - 1) * s.mul_ld;
}

// sin and cos of 2 pi r, |r| <= 1/2: the nearest quarter turn apart, then the Taylor polynomials on an eighth of a turn to
// either side (their remainders are below 2e-9)
__device__ __forceinline__ float2 sin_cos_turns(double r) {
    const double quarter = rint(r * 4.0);
    const float z = float((r - quarter * 0.25) * 6.283185307179586476925286766559), z2 = z * z;
    const int q = int(quarter);
    float s = 2.75573192e-6f, c = -2.75573192e-7f;
    s = __builtin_fmaf(s, z2, -1.98412698e-4f);
    s = __builtin_fmaf(s, z2, 8.33333333e-3f);
    s = __builtin_fmaf(s, z2, -1.66666667e-1f);
    s = __builtin_fmaf(s * z2, z, z);
    c = __builtin_fmaf(c, z2, 2.48015873e-5f);
    c = __builtin_fmaf(c, z2, -1.38888889e-3f);
    c = __builtin_fmaf(c, z2, 4.16666667e-2f);
    c = __builtin_fmaf(c, z2, -0.5f);
    c = __builtin_fmaf(c, z2, 1.0f);
    const float a = q & 1 ? c : s, b = q & 1 ? s : c;  // sin(z + q pi/2) = s, c, -s, -c; cos = c, -s, -c, s
    return make_float2(q & 2 ? -a : a, (q + 1) & 2 ? -b : b);
}

// A workgroup of 256: row t of the stream, a token's embedding at position p.  A thread takes pairs of channels, eight at
// a time, all their loads under way together.
template <typename T>
__device__ __forceinline__ void embed_row(const RmiEmbed &e, uint32_t token, uint32_t p, uint32_t t) {
    if (token >= e.vocab) token = e.vocab - 1;  // ids are validated on the host; never read outside the table
    const T *row = static_cast<const T *>(e.table) + size_t(token) * e.ld;
    const uint32_t pairs = (e.n + 1) / 2;
    for (uint32_t i0 = threadIdx.x; i0 < pairs; i0 += 8 * 256) {
        double turns[8];
        float2 v[8];
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) {
            const uint32_t i = i0 + j * 256 < pairs ? i0 + j * 256 : i0;
            turns[j] = e.turns ? e.turns[i] : 0.0;
            v[j] = make_float2(to_f32(row[2 * i]), to_f32(row[2 * i + 1 < e.n ? 2 * i + 1 : 2 * i]));
        }
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) {
            const uint32_t i = i0 + j * 256;
            if (i >= pairs) break;
            v[j].x *= e.scale;
            v[j].y *= e.scale;
            if (e.turns) {
                const double r = double(p) * turns[j];
                const float2 sc = sin_cos_turns(r - rint(r));  // the whole turns leave in f64
                v[j].x += sc.x;
                v[j].y += sc.y;
            }
            float *dst = e.x + size_t(t) * e.n + 2 * i, *also = e.x_also ? e.x_also + size_t(t) * e.n + 2 * i : nullptr;
            dst[0] = v[j].x;
            if (also) also[0] = v[j].x;
            if (2 * i + 1 < e.n) {
                dst[1] = v[j].y;
                if (also) also[1] = v[j].y;
            }
        }
    }
}

// ---- a product's input (RmiInput) in the registers of a workgroup of 256: R quads of values a thread, quad j of
// thread t at 4 (t + 256 j)
__device__ __forceinline__ float block_sum_f32(float v, float *red) {  // red: four floats of this sum's own
    v = wave_sum_f32(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}
template <int NORM, bool ADD, int R>
struct InputRow {
    f32x4 v[R];
    f32x4 w[NORM != kNormNone ? R : 1], y[ADD ? R : 1], yw[ADD ? R : 1];

    static __device__ __forceinline__ f32x4 quad(const float *p, uint32_t i, uint32_t n, bool quads) {
        if (quads) return *reinterpret_cast<const f32x4 *>(p + (i < n ? i : n - 4));
        f32x4 r;
#pragma unroll
        for (uint32_t e = 0; e < 4; e++) r[e] = p[i + e < n ? i + e : n - 1];
        return r;
    }
    // all loads, none waited for
    __device__ __forceinline__ void load(const RmiInput &in, uint32_t row) {
        const bool quads = (in.n & 3) == 0;
#pragma unroll
        for (int j = 0; j < R; j++) {
            const uint32_t i = (threadIdx.x + j * 256) * 4;
            v[j] = quad(in.x + size_t(row) * in.n, i, in.n, quads);
            if constexpr (ADD) {
                y[j] = quad(in.y + size_t(row) * in.n, i, in.n, quads);
                yw[j] = quad(in.y_weight, i, in.n, quads);
            }
            if constexpr (NORM != kNormNone) w[j] = quad(in.weight, i, in.n, quads);
        }
    }
    // v = the operand, zero past its end; write: v before the norm goes to x_out.  red: twelve floats of LDS
    __device__ __forceinline__ void finish(const RmiInput &in, uint32_t row, bool write, float *red) {
        const float n = float(in.n);
        if constexpr (ADD) {
            float sq = 0.0f;
#pragma unroll
            for (int j = 0; j < R; j++)
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if ((threadIdx.x + j * 256) * 4 + e < in.n) sq = __builtin_fmaf(y[j][e], y[j][e], sq);
            const float r = 1.0f / sqrtf(block_sum_f32(sq, red) / n + in.y_eps);
#pragma unroll
            for (int j = 0; j < R; j++)
#pragma unroll
                for (int e = 0; e < 4; e++) v[j][e] = __builtin_fmaf(y[j][e] * r, yw[j][e], v[j][e]);
        }
#pragma unroll
        for (int j = 0; j < R; j++) {
            const uint32_t i = (threadIdx.x + j * 256) * 4;
            if (ADD && write) {
                float *dst = in.x_out + size_t(row) * in.n + i;
                if ((in.n & 3) == 0) {
                    if (i < in.n) *reinterpret_cast<f32x4 *>(dst) = v[j];
                } else {
#pragma unroll
                    for (uint32_t e = 0; e < 4; e++)
                        if (i + e < in.n) dst[e] = v[j][e];
                }
            }
#pragma unroll
            for (uint32_t e = 0; e < 4; e++)
                if (i + e >= in.n) v[j][e] = 0.0f;
        }
        if constexpr (NORM == kNormLayer) {
            float sum = 0.0f;
#pragma unroll
            for (int j = 0; j < R; j++) sum += (v[j][0] + v[j][1]) + (v[j][2] + v[j][3]);
            const float mean = block_sum_f32(sum, red + 4) / n;
#pragma unroll
            for (int j = 0; j < R; j++)
#pragma unroll
                for (uint32_t e = 0; e < 4; e++) v[j][e] = (threadIdx.x + j * 256) * 4 + e < in.n ? v[j][e] - mean : 0.0f;
        }
        if constexpr (NORM != kNormNone) {
            float sq = 0.0f;
#pragma unroll
            for (int j = 0; j < R; j++)
#pragma unroll
                for (int e = 0; e < 4; e++) sq = __builtin_fmaf(v[j][e], v[j][e], sq);
            const float r = 1.0f / sqrtf(block_sum_f32(sq, red + 8) / n + in.eps);
#pragma unroll
            for (int j = 0; j < R; j++) v[j] = v[j] * r * w[j];
        }
    }
    // the operand as T to dst[0 .. k), k a multiple of 256
    template <typename T>
    __device__ __forceinline__ void store(const RmiInput &in, uint32_t row, T *dst, uint32_t k) {
        const uint32_t k1 = in.x2 ? in.k2 : k;
#pragma unroll
        for (int j = 0; j < R; j++) {
            const uint32_t i = (threadIdx.x + j * 256) * 4;
            if (i < k1) store4(dst + i, v[j]);
        }
        for (uint32_t i = (threadIdx.x + R * 256) * 4; i < k1; i += 1024) store4(dst + i, f32x4{0.f, 0.f, 0.f, 0.f});
        if (!in.x2) return;
        const float *x2 = in.x2 + size_t(row) * in.n2;
        for (uint32_t i = threadIdx.x * 4; i < k - k1; i += 1024) {
            f32x4 b = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (uint32_t e = 0; e < 4; e++)
                if (i + e < in.n2) b[e] = x2[i + e];
            store4(dst + k1 + i, b);
        }
    }
};

#endif  // RMI_DEVICE_DENSE_H
