// Products of one token on dense bf16 / f32 weights, with the input (norms) in their prologue and the layer's
// elementwise work in their epilogue.
#include "dense_launch.h"

namespace {

// The activation sits in LDS, zero past its end, so that a piece past the end of a row (the last one is read again)
// counts for nothing.  Its loads go out before the weights': memory returns in order, and everything waits for it.
constexpr uint32_t kGemvLdsMax = kLdsAskedFor;
constexpr uint32_t kGemvRound = 256;  // LDS activations are padded to this many pieces
template <typename T>
__host__ __device__ inline uint32_t gemv_lds_pieces(uint32_t k_pad) {
    const uint32_t pieces = k_pad / (16 / sizeof(T));
    return (pieces + kGemvRound - 1) / kGemvRound * kGemvRound;
}

struct GemvProblem {
    const void *w;
    uint32_t k_pad, ld;
    uint32_t blocks;  // workgroups of the first of two problems
    RmiInput in;
    RmiRowSegs rs;
};
struct GemvPair {
    GemvProblem p[2];
};

// A wave takes ROWS weight rows, its lanes the pieces of a row, two rounds of 64 in flight; R: quads of the input a
// thread keeps (n <= 1024 R).
template <typename T, int NORM, bool ADD, int ROWS, int R>
__device__ __forceinline__ void gemv_block(const GemvProblem &p, uint32_t block, u32x4 *act, float *red) {
    const uint32_t tid = threadIdx.x, lane = tid & 63, k_pad = p.k_pad;
    const uint32_t row0 = (block * 4 + uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6)))) * ROWS;
    const uint32_t pieces = k_pad / kPieceElems<T>, padded = gemv_lds_pieces<T>(k_pad);
    const T *w = static_cast<const T *>(p.w);
    const RmiRowSegs &rs = p.rs;
    InputRow<NORM, ADD, R> in;
    in.load(p.in, 0);
    const u32x4 *src[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const uint32_t row = row0 + r < rs.n_rows ? row0 + r : rs.n_rows - 1;
        src[r] = reinterpret_cast<const u32x4 *>(w + size_t(row) * p.ld);
    }
    u32x4 cur[2][ROWS];
    auto load = [&](uint32_t p0) {
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const uint32_t at = p0 + u * 64 + lane;
#pragma unroll
            for (int r = 0; r < ROWS; r++) cur[u][r] = src[r][at < pieces ? at : pieces - 1];
        }
    };
    load(0);
    const RmiRowSeg seg = rs.s[seg_of(rs, row0)];
    in.finish(p.in, 0, p.in.x_out && block == 0, red);
    in.store(p.in, 0, reinterpret_cast<T *>(act), padded * kPieceElems<T>);
    __syncthreads();
    float acc[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = 0.0f;
    for (uint32_t p0 = 0; p0 < pieces; p0 += 128) {
        u32x4 now[2][ROWS];
#pragma unroll
        for (int u = 0; u < 2; u++)
#pragma unroll
            for (int r = 0; r < ROWS; r++) now[u][r] = cur[u][r];
        if (p0 + 128 < pieces) load(p0 + 128);
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const u32x4 hv = act[p0 + u * 64 + lane];
#pragma unroll
            for (int r = 0; r < ROWS; r++) acc[r] = dot_piece<T>(now[u][r], hv, acc[r]);
        }
    }
    float mine = 0.0f;
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const float s = wave_sum_f32(acc[r]);
        if (lane == uint32_t(r)) mine = s;
    }
    uint32_t at = row0 + lane - seg.row0;
    float o;
    bool mine_to_store = lane < ROWS && row0 + lane < rs.n_rows && at < seg.n;
    if (ROWS % 2 == 0 && seg.act == kActReluGlu) {  // (gate, up) pairs in neighbouring lanes
        o = fmaxf(mine, 0.0f) * dpp_f32<kDppQuadXor1>(mine);
        mine_to_store = mine_to_store && (lane & 1) == 0;
        at >>= 1;
    } else {
        if (!mine_to_store) return;
        o = apply_act<T>(seg.act, mine, seg.bias ? seg.bias[at] : 0.0f, seg.lower ? seg.lower[at] : 0.0f);
        if (seg.mul) o *= to_f32(mul_row<T>(seg, 0)[at]);
    }
    if (!mine_to_store) return;
    if (seg.out_elem)
        static_cast<T *>(seg.y)[at] = from_f32<T>(o);
    else
        static_cast<float *>(seg.y)[at] = o;
}

template <typename T, int NORM, bool ADD, int ROWS, int R>
__global__ __launch_bounds__(256) void input_gemv_kernel(GemvProblem p) {
    extern __shared__ u32x4 act[];
    __shared__ float red[12];
    gemv_block<T, NORM, ADD, ROWS, R>(p, blockIdx.x, act, red);
}
template <typename T, int NORM, int ROWS, int R>
__global__ __launch_bounds__(256) void input_gemv_pair_kernel(GemvPair p) {
    extern __shared__ u32x4 act[];
    __shared__ float red[12];
    const uint32_t second = blockIdx.x >= p.p[0].blocks ? 1u : 0u;
    gemv_block<T, NORM, false, ROWS, R>(p.p[second], second ? blockIdx.x - p.p[0].blocks : blockIdx.x, act, red);
}

// A workgroup takes ROWS rows, each wave a quarter of their columns, so that a long row is in flight at once; the
// waves' sums meet in LDS.  A lane's products count with the gate and scale of the column segment its piece lies in.
template <typename T, int ROWS>
__global__ __launch_bounds__(256) void gemv_residual_kernel(const T *__restrict__ w, uint32_t k_pad, uint32_t ld, const T *__restrict__ a,
                                                            RmiColSegs cs, float *__restrict__ x, uint32_t width) {
    constexpr int U = 4;
    __shared__ float part[4][ROWS];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6)));
    const uint32_t row0 = blockIdx.x * ROWS;
    const uint32_t pieces = k_pad / kPieceElems<T>, per_wave = ((pieces + 3) / 4 + 63) / 64 * 64;
    const uint32_t p_begin = wave * per_wave, p_end = p_begin + per_wave < pieces ? p_begin + per_wave : pieces;
    const u32x4 *src[ROWS], *hsrc = reinterpret_cast<const u32x4 *>(a);
    float gate[ROWS][kMaxColSegs];
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const uint32_t row = row0 + r < width ? row0 + r : width - 1;
        src[r] = reinterpret_cast<const u32x4 *>(w + size_t(row) * ld);
#pragma unroll
        for (uint32_t i = 0; i < kMaxColSegs; i++) gate[r][i] = i < cs.n_segs ? (cs.s[i].gate ? cs.s[i].gate[row] : 1.0f) * cs.s[i].scale : 0.0f;
    }
    float acc[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = 0.0f;
    u32x4 cur[U][ROWS], hcur[U];
    auto load = [&](uint32_t p0) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const uint32_t p = p0 + u * 64 + lane, pc = p < p_end ? p : pieces - 1;
            hcur[u] = hsrc[pc];
#pragma unroll
            for (int r = 0; r < ROWS; r++) cur[u][r] = src[r][pc];
        }
    };
    if (p_begin < p_end) load(p_begin);
    for (uint32_t p0 = p_begin; p0 < p_end; p0 += 64 * U) {
        u32x4 now[U][ROWS], hv[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            hv[u] = hcur[u];
#pragma unroll
            for (int r = 0; r < ROWS; r++) now[u][r] = cur[u][r];
        }
        if (p0 + 64 * U < p_end) load(p0 + 64 * U);
#pragma unroll
        for (int u = 0; u < U; u++) {
            const uint32_t p = p0 + u * 64 + lane, k = p * kPieceElems<T>;
            const bool live = p < p_end;
#pragma unroll
            for (int r = 0; r < ROWS; r++) {
                float f = gate[r][0];
#pragma unroll
                for (uint32_t i = 0; i + 1 < kMaxColSegs; i++) f = i + 1 < cs.n_segs && k >= cs.s[i].k_end ? gate[r][i + 1] : f;
                const float d = dot_piece<T>(now[u][r], hv[u], 0.0f);
                acc[r] = __builtin_fmaf(f, live ? d : 0.0f, acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const float t = wave_sum_f32(acc[r]);
        if (lane == 0) part[wave][r] = t;
    }
    __syncthreads();
    if (tid < ROWS && row0 + tid < width) x[row0 + tid] += (part[0][tid] + part[1][tid]) + (part[2][tid] + part[3][tid]);
}

GemvProblem problem_of(const RmiDense &w, const RmiInput &in, const RmiRowSegs &segs, uint32_t rows) {
    return GemvProblem{w.data, w.k_pad, w.ld, (w.n_rows + 4 * rows - 1) / (4 * rows), in, segs};
}

template <typename T>
int gemv(const RmiDense &w, const RmiInput &in, const RmiRowSegs &segs, hipStream_t st) {
    const size_t lds = size_t(gemv_lds_pieces<T>(w.k_pad)) * 16;
    // A wave takes four rows; fewer where that would leave compute units with little to do (the prologue, which every
    // workgroup repeats, then weighs less than the wait for memory).  Pairs of rows stay together.
    const uint32_t cus = uint32_t(rmi_device_cus()), pairs = rmi_epilogue_of(segs) == kRowsPaired ? 2 : 1;
    const uint32_t rows = in.norm == kNormRms || w.n_rows > 64 * cus ? 4 : w.n_rows > 4 * cus ? 2 : pairs;
    const GemvProblem p = problem_of(w, in, segs, rows);
    auto go = [&](auto kernel) {
        const int rc = rmi_allow_lds(kernel, lds);
        if (rc == RMI_HIP_OK) hipLaunchKernelGGL(kernel, dim3(p.blocks), dim3(256), lds, st, p);
        return rc;
    };
    const int rc = rmi_input_dispatch(in, [&](auto norm, auto add, auto r) {
        if constexpr (norm.value != kNormRms && (!add.value || r.value <= 4)) {
            if (rows == 1) return go(input_gemv_kernel<T, norm.value, add.value, 1, r.value>);
            if (rows == 2) return go(input_gemv_kernel<T, norm.value, add.value, 2, r.value>);
        }
        if constexpr (!add.value || r.value <= 4)
            return go(input_gemv_kernel<T, norm.value, add.value, 4, r.value>);
        else
            return rmi_fail(RMI_HIP_E_INVALID, "too many values to add in front of a product");
    });
    if (rc != RMI_HIP_OK) return rc;
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

template <typename T>
int gemv_pair(const GemvPair &p, hipStream_t st) {
    const uint32_t k = p.p[0].k_pad > p.p[1].k_pad ? p.p[0].k_pad : p.p[1].k_pad, n = p.p[0].in.n > p.p[1].in.n ? p.p[0].in.n : p.p[1].in.n;
    const size_t lds = size_t(gemv_lds_pieces<T>(k)) * 16;
    auto go = [&](auto kernel) {
        const int rc = rmi_allow_lds(kernel, lds);
        if (rc == RMI_HIP_OK) hipLaunchKernelGGL(kernel, dim3(p.p[0].blocks + p.p[1].blocks), dim3(256), lds, st, p);
        return rc;
    };
    const int rc = n <= 1024 ? go(input_gemv_pair_kernel<T, kNormRms, 4, 1>) : go(input_gemv_pair_kernel<T, kNormRms, 4, 4>);
    if (rc != RMI_HIP_OK) return rc;
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

template <typename T>
int gemv_residual(const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width, hipStream_t st) {
    constexpr int kRows = 2;
    hipLaunchKernelGGL((gemv_residual_kernel<T, kRows>), dim3((width + kRows - 1) / kRows), dim3(256), 0, st,
                       static_cast<const T *>(w.data), w.k_pad, w.ld, static_cast<const T *>(a), segs, x, width);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int check_gemv(uint32_t elem_bytes, const RmiDense &w, const RmiInput &in, const RmiRowSegs &segs) {
    int rc = rmi_check_input(in, w.k_pad, false);
    if (rc == RMI_HIP_OK) rc = rmi_check_row_segs(elem_bytes, w, segs);
    if (rc != RMI_HIP_OK) return rc;
    if (!rmi_dense_gemv_fits(elem_bytes, w.k_pad)) return rmi_fail(RMI_HIP_E_INVALID, "%u columns exceed what the GEMV holds", w.k_pad);
    if (in.y && in.n > kGemvAddMax) return rmi_fail(RMI_HIP_E_INVALID, "%u values to add in front of a product of one token", in.n);
    if (in.x_out && (in.x_out == in.x || in.x_out == in.y)) return rmi_fail(RMI_HIP_E_INVALID, "a product of one token reads and writes x");
    for (uint32_t i = 0; i < segs.n_segs; i++)
        if (segs.s[i].y == in.x || segs.s[i].y == in.y || segs.s[i].y == in.x2)
            return rmi_fail(RMI_HIP_E_INVALID, "a product of one token writes its own input");
    return RMI_HIP_OK;
}

}  // namespace

bool rmi_dense_gemv_fits(uint32_t elem_bytes, uint32_t k_pad) {
    const size_t lds = size_t(elem_bytes == 2 ? gemv_lds_pieces<rmi_bf16>(k_pad) : gemv_lds_pieces<float>(k_pad)) * 16;
    return lds <= kGemvLdsMax && k_pad <= kInputMax;
}

int rmi_dense_gemv(uint32_t elem_bytes, const RmiDense &w, const RmiInput &in, const RmiRowSegs &segs, hipStream_t st) {
    const int rc = check_gemv(elem_bytes, w, in, segs);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? gemv<rmi_bf16>(w, in, segs, st) : gemv<float>(w, in, segs, st);
}

int rmi_dense_gemv_pair(uint32_t elem_bytes, const RmiDense &w0, const RmiInput &in0, const RmiRowSegs &segs0, const RmiDense &w1,
                        const RmiInput &in1, const RmiRowSegs &segs1, hipStream_t st) {
    const bool side_by_side = in0.norm == kNormRms && in1.norm == kNormRms && !in0.y && !in1.y && in0.n <= 4096 && in1.n <= 4096;
    if (!side_by_side) {
        const int rc = rmi_dense_gemv(elem_bytes, w0, in0, segs0, st);
        return rc == RMI_HIP_OK ? rmi_dense_gemv(elem_bytes, w1, in1, segs1, st) : rc;
    }
    int rc = check_gemv(elem_bytes, w0, in0, segs0);
    if (rc == RMI_HIP_OK) rc = check_gemv(elem_bytes, w1, in1, segs1);
    if (rc != RMI_HIP_OK) return rc;
    const GemvPair p{{problem_of(w0, in0, segs0, 4), problem_of(w1, in1, segs1, 4)}};
    return elem_bytes == 2 ? gemv_pair<rmi_bf16>(p, st) : gemv_pair<float>(p, st);
}

int rmi_dense_gemv_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            hipStream_t st) {
    const int rc = rmi_check_col_segs(elem_bytes, w, segs, width);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? gemv_residual<rmi_bf16>(w, a, segs, x, width, st) : gemv_residual<float>(w, a, segs, x, width, st);
}
