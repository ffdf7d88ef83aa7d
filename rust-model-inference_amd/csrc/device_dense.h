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

// What a row segment of a product does with its result z.
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

#endif  // RMI_DEVICE_DENSE_H
