// Products on dense bf16 / f32 weights: a tiled matrix-core GEMM for several tokens, a GEMV for one, each with the
// layer's elementwise work in its epilogue (activations, forget gates, gated residual) and, in the GEMV, the RMS
// norm in its prologue.
#include "device_dense.h"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void norm_kernel(const float *__restrict__ x, const uint32_t *__restrict__ rows,
                                                   const float *__restrict__ weight, float eps, T *__restrict__ h, uint32_t n,
                                                   uint32_t k_pad, uint32_t ld) {
    __shared__ float red[4];
    const uint32_t tid = threadIdx.x;
    x += size_t(rows ? rows[blockIdx.x] : blockIdx.x) * n;
    h += size_t(blockIdx.x) * ld;
    float sq = 0.0f;
    for (uint32_t i = tid; i < n; i += 256) sq = __builtin_fmaf(x[i], x[i], sq);
    sq = wave_sum_f32(sq);
    if ((tid & 63) == 0) red[tid >> 6] = sq;
    __syncthreads();
    const float r = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / float(n) + eps);
    for (uint32_t i = tid; i < k_pad; i += 256) h[i] = from_f32<T>(i < n ? x[i] * r * weight[i] : 0.0f);
}

template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(const T *__restrict__ table, uint32_t ld, const uint32_t *__restrict__ tok,
                                                    uint32_t vocab, float scale, float *__restrict__ x, uint32_t n) {
    uint32_t t = tok[blockIdx.x];
    if (t >= vocab) t = vocab - 1;  // ids are validated on the host; never read outside the table
    for (uint32_t i = threadIdx.x; i < n; i += 256) x[size_t(blockIdx.x) * n + i] = to_f32(table[size_t(t) * ld + i]) * scale;
}

// which row segment a row lies in: the starts sit side by side (unused ones at the end of the range)
__device__ __forceinline__ uint32_t seg_of(const RmiRowSegs &rs, uint32_t row) {
    uint32_t si = 0;
#pragma unroll
    for (uint32_t i = 1; i < kMaxRowSegs; i++) si += row >= rs.start[i] ? 1u : 0u;
    return si;
}

// ------------------------------------------------------------------ GEMM
// One workgroup of four waves: BN weight rows x BT tokens, k in steps of 128 bytes a row through two LDS buffers; the
// pieces of the next PD steps are on their way to registers while one is multiplied.  The largest tile keeps one LDS
// buffer (NB = 1), so that three workgroups share a compute unit.  A row of a buffer is eight
// 16-byte pieces, piece p at slot p ^ (row & 7), so that the sixteen rows of a fragment spread over the banks.
// Weights are the A operand: a lane ends with four consecutive rows of one token.
constexpr uint32_t kStepBytes = 128;

template <typename T, int BN, int BT, int WN, int WT, int PD, int NB, int WPS, bool RESIDUAL>
__global__ __launch_bounds__(256, WPS) void dense_gemm_kernel(const T *__restrict__ w, const T *__restrict__ a, uint32_t n_rows,
                                                              uint32_t k_pad, uint32_t ld, uint32_t n_tokens, uint32_t grid_n, uint32_t grid_t, uint32_t xcd_split,
                                                         RmiRowSegs rs, RmiColSegs cs, float *__restrict__ x, uint32_t width) {
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
                            if (s.gate) v *= *reinterpret_cast<const f32x4 *>(s.gate + at);
                            *reinterpret_cast<f32x4 *>(x + at) += v;
                        } else {
#pragma unroll
                            for (int r = 0; r < 4; r++)
                                if (row + r < width) x[at + r] += acc[i][j][r] * s.scale * (s.gate ? s.gate[at + r] : 1.0f);
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
#pragma unroll
            for (int r = 0; r < 4; r++) {
                bias[r] = s.bias && r0 + r < s.n ? s.bias[r0 + r] : 0.0f;
                lower[r] = s.lower && r0 + r < s.n ? s.lower[r0 + r] : 0.0f;
            }
#pragma unroll
            for (int j = 0; j < NT; j++) {
                const uint32_t tok = tok0 + wt + j * 16 + fr;
                f32x4 o;
#pragma unroll
                for (int r = 0; r < 4; r++) o[r] = apply_act<T>(s.act, acc[i][j][r], bias[r], lower[r]);
                if (tok >= n_tokens) continue;
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

template <typename T, bool RESIDUAL>
int launch_gemm(const RmiDense &w, const void *a, const RmiRowSegs &rs, const RmiColSegs &cs, float *x, uint32_t width,
                uint32_t n_tokens, hipStream_t st) {
    const uint32_t n_rows = RESIDUAL ? width : w.n_rows;
    auto go = [&](auto kernel, uint32_t bn, uint32_t bt) {
        const uint32_t gn = (n_rows + bn - 1) / bn, gt = (n_tokens + bt - 1) / bt;
        const uint32_t split = rmi_gemm_xcd_split(gn, gt, double(n_rows) * w.k_pad, double(n_tokens) * w.k_pad);
        hipLaunchKernelGGL(kernel, dim3(gn * gt), dim3(256), 0, st, static_cast<const T *>(w.data), static_cast<const T *>(a), n_rows,
                           w.k_pad, w.ld, n_tokens, gn, gt, split, rs, cs, x, width);
    };
    const uint64_t cus = uint64_t(rmi_device_cus());
    auto tiles = [&](uint32_t bn, uint32_t bt) { return uint64_t((n_rows + bn - 1) / bn) * ((n_tokens + bt - 1) / bt); };
    if (n_tokens <= 16)
        go(dense_gemm_kernel<T, 64, 16, 16, 16, 4, 2, 4, RESIDUAL>, 64, 16);
    else if (tiles(128, 128) >= 2 * cus)
        go(dense_gemm_kernel<T, 128, 128, 64, 64, 1, 1, 3, RESIDUAL>, 128, 128);
    else if (tiles(64, 64) >= cus)
        go(dense_gemm_kernel<T, 64, 64, 32, 32, 4, 2, 4, RESIDUAL>, 64, 64);
    else
        go(dense_gemm_kernel<T, 64, 32, 32, 16, 4, 2, 4, RESIDUAL>, 64, 32);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

// ------------------------------------------------------------------ GEMV
// The activation sits in LDS, zero past its end, so that a piece past the end of a row (the last one is read again)
// counts for nothing.  Its loads go out before the weights': memory returns in order, and everything waits for it.
constexpr uint32_t kGemvLdsMax = kLdsAskedFor;
constexpr uint32_t kGemvRound = 256;  // LDS activations are padded to this many pieces
template <typename T>
__host__ __device__ inline uint32_t gemv_lds_pieces(uint32_t k_pad) {
    const uint32_t pieces = k_pad / (16 / sizeof(T));
    return (pieces + kGemvRound - 1) / kGemvRound * kGemvRound;
}

// A wave takes ROWS weight rows, its lanes the pieces of a row, two rounds of 64 in flight; R: quads of x a thread
// keeps (n <= 1024 R).
template <typename T, int ROWS, int R>
__global__ __launch_bounds__(256) void norm_gemv_kernel(const T *__restrict__ w, uint32_t k_pad, uint32_t ld, const float *__restrict__ x,
                                                        const float *__restrict__ weight, float eps, uint32_t n, RmiRowSegs rs) {
    extern __shared__ u32x4 act[];
    __shared__ float red[4];
    const uint32_t tid = threadIdx.x, lane = tid & 63;
    const uint32_t row0 = (blockIdx.x * 4 + uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6)))) * ROWS;
    const uint32_t pieces = k_pad / kPieceElems<T>, padded = gemv_lds_pieces<T>(k_pad);
    f32x4 xv[R], nv[R];
    const bool quads = (n & 3) == 0;
#pragma unroll
    for (int j = 0; j < R; j++) {
        const uint32_t i = (tid + j * 256) * 4;
        if (quads) {
            const uint32_t ic = i < n ? i : n - 4;
            xv[j] = *reinterpret_cast<const f32x4 *>(x + ic);
            nv[j] = *reinterpret_cast<const f32x4 *>(weight + ic);
        } else {
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const uint32_t ic = i + e < n ? i + e : n - 1;
                xv[j][e] = x[ic];
                nv[j][e] = weight[ic];
            }
        }
    }
    const u32x4 *src[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) {
        const uint32_t row = row0 + r < rs.n_rows ? row0 + r : rs.n_rows - 1;
        src[r] = reinterpret_cast<const u32x4 *>(w + size_t(row) * ld);
    }
    u32x4 cur[2][ROWS];
    auto load = [&](uint32_t p0) {
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const uint32_t p = p0 + u * 64 + lane;
#pragma unroll
            for (int r = 0; r < ROWS; r++) cur[u][r] = src[r][p < pieces ? p : pieces - 1];
        }
    };
    load(0);
    const RmiRowSeg seg = rs.s[seg_of(rs, row0)];
    float sq = 0.0f;
#pragma unroll
    for (int j = 0; j < R; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            if ((tid + j * 256) * 4 + e >= n) xv[j][e] = 0.0f;
            sq = __builtin_fmaf(xv[j][e], xv[j][e], sq);
        }
    sq = wave_sum_f32(sq);
    if (lane == 0) red[tid >> 6] = sq;
    __syncthreads();
    const float scale = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / float(n) + eps);
    T *h = reinterpret_cast<T *>(act);
    const uint32_t h_elems = padded * kPieceElems<T>;  // a multiple of 1024
#pragma unroll
    for (int j = 0; j < R; j++) {
        const uint32_t i = (tid + j * 256) * 4;
        if (i < h_elems) store4(h + i, xv[j] * scale * nv[j]);
    }
    for (uint32_t i = (tid + R * 256) * 4; i < h_elems; i += 1024) store4(h + i, f32x4{0.f, 0.f, 0.f, 0.f});
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
    const uint32_t at = row0 + lane - seg.row0;
    if (lane >= ROWS || row0 + lane >= rs.n_rows || at >= seg.n) return;
    const float o = apply_act<T>(seg.act, mine, seg.bias ? seg.bias[at] : 0.0f, seg.lower ? seg.lower[at] : 0.0f);
    if (seg.out_elem)
        static_cast<T *>(seg.y)[at] = from_f32<T>(o);
    else
        static_cast<float *>(seg.y)[at] = o;
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

constexpr uint32_t kNormGemvMaxN = 16384;  // what a workgroup keeps of x in registers

template <typename T, int R>
int norm_gemv_r(const RmiDense &w, const float *x, const float *weight, float eps, uint32_t n, const RmiRowSegs &segs, hipStream_t st) {
    const size_t lds = size_t(gemv_lds_pieces<T>(w.k_pad)) * 16;
    constexpr int kRows = 4;
    const int rc = rmi_allow_lds(norm_gemv_kernel<T, kRows, R>, lds);
    if (rc != RMI_HIP_OK) return rc;
    hipLaunchKernelGGL((norm_gemv_kernel<T, kRows, R>), dim3((w.n_rows + 4 * kRows - 1) / (4 * kRows)), dim3(256), lds, st,
                       static_cast<const T *>(w.data), w.k_pad, w.ld, x, weight, eps, n, segs);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}
template <typename T>
int norm_gemv(const RmiDense &w, const float *x, const float *weight, float eps, uint32_t n, const RmiRowSegs &segs, hipStream_t st) {
    if (!rmi_dense_gemv_fits(sizeof(T), w.k_pad)) return rmi_fail(RMI_HIP_E_INVALID, "%u columns exceed what the GEMV holds", w.k_pad);
    if (n <= 1024) return norm_gemv_r<T, 1>(w, x, weight, eps, n, segs, st);
    if (n <= 4096) return norm_gemv_r<T, 4>(w, x, weight, eps, n, segs, st);
    return norm_gemv_r<T, 16>(w, x, weight, eps, n, segs, st);
}

template <typename T>
int gemv_residual(const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width, hipStream_t st) {
    constexpr int kRows = 2;
    hipLaunchKernelGGL((gemv_residual_kernel<T, kRows>), dim3((width + kRows - 1) / kRows), dim3(256), 0, st,
                       static_cast<const T *>(w.data), w.k_pad, w.ld, static_cast<const T *>(a), segs, x, width);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

}  // namespace

int rmi_dense_norm(uint32_t elem_bytes, const float *x, const uint32_t *rows, const float *weight, float eps, void *h,
                   uint32_t n_tokens, uint32_t n, uint32_t k_pad, hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    if (elem_bytes == 2)
        hipLaunchKernelGGL(norm_kernel<rmi_bf16>, dim3(n_tokens), dim3(256), 0, st, x, rows, weight, eps, static_cast<rmi_bf16 *>(h), n, k_pad, rmi_dense_ld(k_pad, 2));
    else
        hipLaunchKernelGGL(norm_kernel<float>, dim3(n_tokens), dim3(256), 0, st, x, rows, weight, eps, static_cast<float *>(h), n, k_pad, rmi_dense_ld(k_pad, 4));
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_dense_embed(uint32_t elem_bytes, const RmiDense &table, const uint32_t *tok, uint32_t vocab, float scale, float *x,
                    uint32_t n_tokens, uint32_t n, hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    if (elem_bytes == 2)
        hipLaunchKernelGGL(embed_kernel<rmi_bf16>, dim3(n_tokens), dim3(256), 0, st, static_cast<const rmi_bf16 *>(table.data), table.ld,
                           tok, vocab, scale, x, n);
    else
        hipLaunchKernelGGL(embed_kernel<float>, dim3(n_tokens), dim3(256), 0, st, static_cast<const float *>(table.data), table.ld, tok,
                           vocab, scale, x, n);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_dense_gemm(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiRowSegs &segs, uint32_t n_tokens, hipStream_t st) {
    if (n_tokens == 0 || w.n_rows == 0) return RMI_HIP_OK;
    if (segs.n_rows != w.n_rows || segs.n_segs == 0 || segs.n_segs > kMaxRowSegs || w.k_pad % kDenseKAlign || w.ld != rmi_dense_ld(w.k_pad, elem_bytes))
        return rmi_fail(RMI_HIP_E_INVALID, "row segments do not fit the weight");
    return elem_bytes == 2 ? launch_gemm<rmi_bf16, false>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st)
                           : launch_gemm<float, false>(w, a, segs, RmiColSegs{}, nullptr, 0, n_tokens, st);
}

static int check_col_segs(uint32_t elem_bytes, const RmiDense &w, const RmiColSegs &segs, uint32_t width) {
    if (w.ld != rmi_dense_ld(w.k_pad, elem_bytes) || segs.n_segs == 0 || segs.n_segs > kMaxColSegs || segs.s[segs.n_segs - 1].k_end != w.k_pad || w.n_rows < width)
        return rmi_fail(RMI_HIP_E_INVALID, "column segments do not fit the weight");
    for (uint32_t i = 0; i < segs.n_segs; i++)
        if (segs.s[i].k_end % kDenseKAlign || segs.s[i].k_end <= (i ? segs.s[i - 1].k_end : 0u))
            return rmi_fail(RMI_HIP_E_INVALID, "column segments do not fit the weight");
    return RMI_HIP_OK;
}

int rmi_dense_gemm_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            uint32_t n_tokens, hipStream_t st) {
    if (n_tokens == 0) return RMI_HIP_OK;
    const int rc = check_col_segs(elem_bytes, w, segs, width);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? launch_gemm<rmi_bf16, true>(w, a, RmiRowSegs{}, segs, x, width, n_tokens, st)
                           : launch_gemm<float, true>(w, a, RmiRowSegs{}, segs, x, width, n_tokens, st);
}

bool rmi_dense_gemv_fits(uint32_t elem_bytes, uint32_t k_pad) {
    const size_t lds = size_t(elem_bytes == 2 ? gemv_lds_pieces<rmi_bf16>(k_pad) : gemv_lds_pieces<float>(k_pad)) * 16;
    return lds <= kGemvLdsMax && k_pad <= kNormGemvMaxN;
}

int rmi_dense_norm_gemv(uint32_t elem_bytes, const RmiDense &w, const float *x, const float *weight, float eps, uint32_t n,
                        const RmiRowSegs &segs, hipStream_t st) {
    if (segs.n_rows != w.n_rows || segs.n_segs == 0 || segs.n_segs > kMaxRowSegs || n > w.k_pad)
        return rmi_fail(RMI_HIP_E_INVALID, "row segments do not fit the weight");
    return elem_bytes == 2 ? norm_gemv<rmi_bf16>(w, x, weight, eps, n, segs, st) : norm_gemv<float>(w, x, weight, eps, n, segs, st);
}

int rmi_dense_gemv_residual(uint32_t elem_bytes, const RmiDense &w, const void *a, const RmiColSegs &segs, float *x, uint32_t width,
                            hipStream_t st) {
    const int rc = check_col_segs(elem_bytes, w, segs, width);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? gemv_residual<rmi_bf16>(w, a, segs, x, width, st) : gemv_residual<float>(w, a, segs, x, width, st);
}
