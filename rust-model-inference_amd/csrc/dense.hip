// Products of several tokens on dense bf16 / f32 weights: the inputs (norms) in front of them, a tiled matrix-core
// GEMM with the layer's elementwise work in its epilogue (activations, gates, gated residual), and the embedding.
#include "dense_launch.h"

namespace {

template <typename T, int NORM, bool ADD, int R>
__global__ __launch_bounds__(256) void input_kernel(RmiInput in, const uint32_t *__restrict__ rows, T *__restrict__ h, uint32_t k_pad,
                                                    uint32_t ld) {
    __shared__ float red[12];
    InputRow<NORM, ADD, R> r;
    const uint32_t row = rows ? rows[blockIdx.x] : blockIdx.x;
    r.load(in, row);
    r.finish(in, row, in.x_out != nullptr, red);
    if (h) r.store(in, row, h + size_t(blockIdx.x) * ld, k_pad);
}

template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(RmiEmbed e, const uint32_t *__restrict__ tok, uint32_t pos0) {
    embed_row<T>(e, tok[blockIdx.x], pos0 + blockIdx.x, blockIdx.x);
}

// ------------------------------------------------------------------ GEMM
// One workgroup of four waves: BN weight rows x BT tokens, k in steps of 128 bytes a row through two LDS buffers; the
// pieces of the next PD steps are on their way to registers while one is multiplied.  The largest tile keeps one LDS
// buffer (NB = 1), so that three workgroups share a compute unit.  A row of a buffer is eight
// 16-byte pieces, piece p at slot p ^ (row & 7), so that the sixteen rows of a fragment spread over the banks.
// Weights are the A operand: a lane ends with four consecutive rows of one token.
constexpr uint32_t kStepBytes = 128;
constexpr int kResidual = -1;  // the epilogue that adds to the residual stream; the others are RmiEpilogue's

template <typename T, int BN, int BT, int WN, int WT, int PD, int NB, int WPS, int EPI>
__global__ __launch_bounds__(256, WPS) void dense_gemm_kernel(const T *__restrict__ w, const T *__restrict__ a, uint32_t n_rows,
                                                              uint32_t k_pad, uint32_t ld, uint32_t n_tokens, uint32_t grid_n, uint32_t grid_t, uint32_t xcd_split,
                                                         RmiRowSegs rs, RmiColSegs cs, float *__restrict__ x, uint32_t width) {
    constexpr bool RESIDUAL = EPI == kResidual;
    static_assert((BN / WN) * (BT / WT) == 4, "four waves");
    static_assert(kDenseKAlign * sizeof(T) % (kStepBytes * PD) == 0, "whole rounds of the register slots");
    constexpr int NN = WN / 16, NT = WT / 16;
    constexpr int PW = BN * 8 / 256, PA = (BT * 8 + 255) / 256;  // pieces a thread loads per step
    __shared__ u32x4 lds[NB][(BN + BT) * 8];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6)));
    uint32_t n_tile, t_tile;
    rmi_gemm_tile_of(blockIdx.x, grid_n, grid_t, 1u, xcd_split, n_tile, t_tile);
    const uint32_t row0 = n_tile * BN, tok0 = t_tile * BT;
    const uint32_t wn = (wave % (BN / WN)) * WN, wt = (wave / (BN / WN)) * WT;
    const size_t stride = size_t(ld) * sizeof(T);

    const uint8_t *wsrc[PW], *asrc[PA];
    uint32_t wdst[PW], adst[PA];
#pragma unroll
    for (int i = 0; i < PW; i++) {
        const uint32_t e = tid + i * 256, r = e >> 3, p = e & 7;
        const uint32_t row = row0 + r < n_rows ? row0 + r : n_rows - 1;  // rows past the end are read again and not stored
        wsrc[i] = reinterpret_cast<const uint8_t *>(w) + row * stride + p * 16;
        wdst[i] = r * 8 + (p ^ (r & 7));
    }
#pragma unroll
    for (int i = 0; i < PA; i++) {
        const uint32_t e = tid + i * 256, r = (e >> 3) % BT, p = e & 7;  // (fewer pieces than threads: some load twice)
        const uint32_t tok = tok0 + r < n_tokens ? tok0 + r : n_tokens - 1;
        asrc[i] = reinterpret_cast<const uint8_t *>(a) + tok * stride + p * 16;
        adst[i] = BN * 8 + r * 8 + (p ^ (r & 7));
    }
    f32x4 acc[NN][NT];
#pragma unroll
    for (int i = 0; i < NN; i++)
#pragma unroll
        for (int j = 0; j < NT; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr uint32_t kStepElems = kStepBytes / sizeof(T);
    const uint32_t n_steps = k_pad / kStepElems;
    u32x4 rw[PD][PW], ra[PD][PA];
    auto load = [&](int slot, uint32_t step) {
        // always issued (past the end the last step again): the waits count loads, and a skipped one would make every
        // wait a wait for all
        step = step < n_steps ? step : n_steps - 1;
#pragma unroll
        for (int i = 0; i < PW; i++) rw[slot][i] = *reinterpret_cast<const u32x4 *>(wsrc[i] + size_t(step) * kStepBytes);
#pragma unroll
        for (int i = 0; i < PA; i++) ra[slot][i] = *reinterpret_cast<const u32x4 *>(asrc[i] + size_t(step) * kStepBytes);
    };
    auto park = [&](int slot, uint32_t buf) {
#pragma unroll
        for (int i = 0; i < PW; i++) lds[buf][wdst[i]] = rw[slot][i];
#pragma unroll
        for (int i = 0; i < PA; i++) lds[buf][adst[i]] = ra[slot][i];
    };
    const uint32_t fr = lane & 15, g = lane >> 4;
    // a finished column segment goes to the residual stream at once (each element is one thread's), so that no second
    // set of accumulators is held
    auto fold = [&](const RmiColSeg &s) {
        if constexpr (RESIDUAL) {
            const bool quads = (width & 3) == 0;
#pragma unroll
            for (int j = 0; j < NT; j++) {
                const uint32_t tok = tok0 + wt + j * 16 + fr;
#pragma unroll
                for (int i = 0; i < NN; i++) {
                    const uint32_t row = row0 + wn + i * 16 + g * 4;
                    const size_t at = size_t(tok) * width + row;
                    if (tok < n_tokens && row < width) {
                        if (quads) {
                            f32x4 v = acc[i][j] * s.scale;
                            if (s.gate) v *= *reinterpret_cast<const f32x4 *>(s.gate + size_t(tok) * s.gate_ld + row);
                            *reinterpret_cast<f32x4 *>(x + at) += v;
                        } else {
#pragma unroll
                            for (int r = 0; r < 4; r++)
                                if (row + r < width) x[at + r] += acc[i][j][r] * s.scale * (s.gate ? s.gate[size_t(tok) * s.gate_ld + row + r] : 1.0f);
                        }
                    }
                    acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
                }
            }
        }
    };
#pragma unroll
    for (int j = 0; j < PD; j++) {
        load(j, j);
        asm volatile("" ::: "memory");  // in this order, and here: the waits in the loop count on it
    }
    park(0, 0);
    load(0, PD);
    asm volatile("" ::: "memory");
    __syncthreads();
    uint32_t step = 0;
    for (uint32_t seg = 0; seg < (RESIDUAL ? cs.n_segs : 1u); seg++) {
        // segments end at multiples of kDenseKAlign, whole rounds of the register slots
        const uint32_t seg_end = RESIDUAL ? cs.s[seg].k_end / kStepElems : n_steps;
        for (; step < seg_end; step += PD) {
#pragma unroll
            for (int j = 0; j < PD; j++) {  // register slots by compile-time index
                const uint32_t buf = (step + j) & (NB - 1);
#pragma unroll
                for (int c = 0; c < 2; c++) {
                    u32x4 fw[NN], fa[NT];
#pragma unroll
                    for (int i = 0; i < NN; i++) {
                        const uint32_t r = wn + i * 16 + fr;
                        fw[i] = lds[buf][r * 8 + ((c * 4 + g) ^ (r & 7))];
                    }
#pragma unroll
                    for (int i = 0; i < NT; i++) {
                        const uint32_t r = wt + i * 16 + fr;
                        fa[i] = lds[buf][BN * 8 + r * 8 + ((c * 4 + g) ^ (r & 7))];
                    }
#pragma unroll
                    for (int i = 0; i < NN; i++)
#pragma unroll
                        for (int i2 = 0; i2 < NT; i2++) acc[i][i2] = mma16<T>(fw[i], fa[i2], acc[i][i2]);
                }
                if (NB == 1) __syncthreads();
                park((j + 1) % PD, buf ^ (NB - 1));  // (behind the last step: that step again, read by nobody)
                load((j + 1) % PD, step + j + 1 + PD);
                __syncthreads();
            }
        }
        if (RESIDUAL) fold(cs.s[seg]);
    }

    if constexpr (!RESIDUAL) {
#pragma unroll
        for (int i = 0; i < NN; i++) {
            const uint32_t tile_row = row0 + wn + i * 16;  // a tile of sixteen rows lies in one segment
            if (tile_row >= n_rows) continue;
            const RmiRowSeg &s = rs.s[seg_of(rs, tile_row)];
            const uint32_t r0 = tile_row - s.row0 + g * 4;
            float bias[4], lower[4];
            if constexpr (EPI == kRowsActed || EPI == kRowsTimesTable) {
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    bias[r] = s.bias && r0 + r < s.n ? s.bias[r0 + r] : 0.0f;
                    lower[r] = s.lower && r0 + r < s.n ? s.lower[r0 + r] : 0.0f;
                }
            }
#pragma unroll
            for (int j = 0; j < NT; j++) {
                const uint32_t tok = tok0 + wt + j * 16 + fr;
                if constexpr (EPI == kRowsPaired) {  // (gate, up) twice: two results
                    if (tok >= n_tokens) continue;
#pragma unroll
                    for (uint32_t r = 0; r < 2; r++) {
                        const float v = fmaxf(acc[i][j][2 * r], 0.0f) * acc[i][j][2 * r + 1];
                        const size_t at = size_t(tok) * s.ld + r0 / 2 + r;
                        if (r0 + 2 * r < s.n) {
                            if (s.out_elem)
                                static_cast<T *>(s.y)[at] = from_f32<T>(v);
                            else
                                static_cast<float *>(s.y)[at] = v;
                        }
                    }
                    continue;
                }
                f32x4 o = acc[i][j];
                if constexpr (EPI == kRowsActed || EPI == kRowsTimesTable) {
#pragma unroll
                    for (int r = 0; r < 4; r++) o[r] = apply_act<T>(s.act, o[r], bias[r], lower[r]);
                }
                if (tok >= n_tokens) continue;
                if constexpr (EPI == kRowsTimesTable) {
                    if (s.mul) {
                        const T *m = mul_row<T>(s, tok) + r0;
#pragma unroll
                        for (uint32_t r = 0; r < 4; r++)
                            if (r0 + r < s.n) o[r] *= to_f32(m[r]);
                    }
                }
                const size_t at = size_t(tok) * s.ld + r0;
                if (r0 + 3 < s.n && (s.ld & 3) == 0) {
                    if (s.out_elem)
                        store4(static_cast<T *>(s.y) + at, o);
                    else
                        store4(static_cast<float *>(s.y) + at, o);
                } else {
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (r0 + r < s.n) {
                            if (s.out_elem)
                                static_cast<T *>(s.y)[at + r] = from_f32<T>(o[r]);
                            else
                                static_cast<float *>(s.y)[at + r] = o[r];
                        }
                }
            }
        }
    }
}

template <typename T, int EPI>
int launch_gemm(const RmiDense &w, const void *a, const RmiRowSegs &rs, const RmiColSegs &cs, float *x, uint32_t width,
                uint32_t n_tokens, hipStream_t st) {
    const uint32_t n_rows = EPI == kResidual ? width : w.n_rows;
    auto go = [&](auto kernel, uint32_t bn, uint32_t bt) {
        const uint32_t gn = (n_rows + bn - 1) / bn, gt = (n_tokens + bt - 1) / bt;
        const uint32_t split = rmi_gemm_xcd_split(gn, gt, double(n_rows) * w.k_pad, double(n_tokens) * w.k_pad);
        hipLaunchKernelGGL(kernel, dim3(gn * gt), dim3(256), 0, st, static_cast<const T *>(w.data), static_cast<const T *>(a), n_rows,
                           w.k_pad, w.ld, n_tokens, gn, gt, split, rs, cs, x, width);
    };
    const uint64_t cus = uint64_t(rmi_device_cus());
    auto tiles = [&](uint32_t bn, uint32_t bt) { return uint64_t((n_rows + bn - 1) / bn) * ((n_tokens + bt - 1) / bt); };
    if (n_tokens <= 16)
        go(dense_gemm_kernel<T, 64, 16, 16, 16, 4, 2, 4, EPI>, 64, 16);
    else if (tiles(128, 128) >= 2 * cus)
        go(dense_gemm_kernel<T, 128, 128, 64, 64, 1, 1, 3, EPI>, 128, 128);
    else if (tiles(64, 64) >= cus)
        go(dense_gemm_kernel<T, 64, 64, 32, 32, 4, 2, 4, EPI>, 64, 64);
    else
        go(dense_gemm_kernel<T, 64, 32, 32, 16, 4, 2, 4, EPI>, 64, 32);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

}  // namespace

int rmi_dense_input(uint32_t elem_bytes, const RmiInput &in, const uint32_t *rows, void *h, uint32_t n_tokens, uint32_t k_pad,
                    hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    int rc = rmi_check_input(in, k_pad, h == nullptr);
    if (rc != RMI_HIP_OK) return rc;
    auto go = [&](auto type) {
        using T = decltype(type);
        return rmi_input_dispatch(in, [&](auto norm, auto add, auto r) {
            hipLaunchKernelGGL((input_kernel<T, norm.value, add.value, r.value>), dim3(n_tokens), dim3(256), 0, st, in, rows, static_cast<T *>(h),
                               k_pad, rmi_dense_ld(k_pad, sizeof(T)));
            return RMI_HIP_OK;
        });
    };
    rc = elem_bytes == 2 ? go(rmi_bf16()) : go(float());
    RMI_HIP_CHECK(hipGetLastError());
    return rc;
}

int rmi_dense_embed(uint32_t elem_bytes, const RmiEmbed &e, const uint32_t *tok, uint32_t pos0, uint32_t n_tokens, hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    if (elem_bytes == 2)
        hipLaunchKernelGGL(embed_kernel<rmi_bf16>, dim3(n_tokens), dim3(256), 0, st, e, tok, pos0);
    else
        hipLaunchKernelGGL(embed_kernel<float>, dim3(n_tokens), dim3(256), 0, st, e, tok, pos0);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_dense_gemm(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiRowSegs &segs, uint32_t n_tokens, hipStream_t st) {
    if (n_tokens == 0 || w.n_rows == 0) return RMI_HIP_OK;
    const int rc = rmi_check_row_segs(elem_bytes, w, segs);
    if (rc != RMI_HIP_OK) return rc;
    auto go = [&](auto type) {
        using T = decltype(type);
        switch (rmi_epilogue_of(segs)) {
            case kRowsActed: return launch_gemm<T, kRowsActed>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st);
            case kRowsPaired: return launch_gemm<T, kRowsPaired>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st);
            case kRowsTimesTable: return launch_gemm<T, kRowsTimesTable>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st);
            default: return launch_gemm<T, kRowsPlain>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st);
        }
    };
    return elem_bytes == 2 ? go(rmi_bf16()) : go(float());
}

int rmi_dense_gemm_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            uint32_t n_tokens, hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    const int rc = rmi_check_col_segs(elem_bytes, w, segs, width);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? launch_gemm<rmi_bf16, kResidual>(w, a, RmiRowSegs{}, segs, x, width, n_tokens, st)
                           : launch_gemm<float, kResidual>(w, a, RmiRowSegs{}, segs, x, width, n_tokens, st);
}
