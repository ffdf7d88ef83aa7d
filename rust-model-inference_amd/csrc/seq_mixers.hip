// Mixers over time (seq_mixers.h): kernels for passes of several tokens and for single tokens.
#include "seq_mixers.h"

#include "device_conv.h"
#include "device_dense.h"

namespace {

// Where key `k` of a block of 32 lies.  The softmax weights of keys 16t + 4g + r come out of the score product in
// register r of lane group g, tile t; the value product's operand wants lane group g's piece contiguous: for bf16 a
// piece is both tiles' four keys, for f32 a piece is one tile's.
template <typename T>
__device__ __forceinline__ uint32_t value_slot(uint32_t k) {
    if (sizeof(T) == 4) return k;
    return ((k >> 2) & 3) * 8 + (k >> 4) * 4 + (k & 3);
}

// ---- convolution, rotation, value norm
// elements 2i, 2i + 1 of a query or key head whose channels start at c0, convolved and rotated
__device__ __forceinline__ void conv_rotate_pair(const ConvCtx &x, const RmiAttnShape &s, const float *cos_t, const float *sin_t,
                                                 uint32_t t, uint32_t pos0, uint32_t c0, uint32_t i, float &a, float &b) {
    a = 2 * i < s.dim ? conv_at(x, t, pos0, c0 + 2 * i) : 0.0f;
    b = 2 * i + 1 < s.dim ? conv_at(x, t, pos0, c0 + 2 * i + 1) : 0.0f;
    if (2 * i < s.rot_dims) {
        const size_t at = size_t(pos0 + t) * (s.rot_dims / 2) + i;
        const float c = cos_t[at], sn = sin_t[at], ra = a;
        a = __builtin_fmaf(ra, c, -(b * sn));
        b = __builtin_fmaf(b, c, ra * sn);
    }
}
template <typename T>
__device__ __forceinline__ void store_pair(T *p, float a, float b);
template <>
__device__ __forceinline__ void store_pair<float>(float *p, float a, float b) {
    p[0] = a;
    p[1] = b;
}
template <>
__device__ __forceinline__ void store_pair<rmi_bf16>(rmi_bf16 *p, float a, float b) {  // p is 4-byte aligned
    *reinterpret_cast<uint32_t *>(p) = uint32_t(f32_to_bf16(a)) | (uint32_t(f32_to_bf16(b)) << 16);
}
// one wave: key head g of token t to its cache row
template <typename T>
__device__ __forceinline__ void key_row(const ConvCtx &x, const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t t, uint32_t g, uint32_t lane) {
    T *row = static_cast<T *>(a.k_cache) + (size_t(g) * s.capacity + (a.pos0 + t) % s.capacity) * s.dk_pad;
    const uint32_t c0 = (s.heads + g) * s.dim;
    for (uint32_t i = lane; i < s.dk_pad / 2; i += 64) {
        float p, q;
        conv_rotate_pair(x, s, a.cos_t, a.sin_t, t, a.pos0, c0, i, p, q);
        store_pair(row + 2 * i, p, q);
    }
}
// one wave: value head g of token t, over its root mean square, to its place in the value block
template <typename T>
__device__ __forceinline__ void value_row(const ConvCtx &x, const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t t, uint32_t g, uint32_t lane) {
    const uint32_t c0 = (s.heads + s.kv_heads) * s.dim + g * s.vdim;
    float v[kMaxHeadDim / 64], sq = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++) {
        const uint32_t d = lane + j * 64;
        v[j] = d < s.vdim ? conv_at(x, t, a.pos0, c0 + d) : 0.0f;
        sq = __builtin_fmaf(v[j], v[j], sq);
    }
    const float r = s.v_norm ? 1.0f / sqrtf(wave_sum_f32(sq) / float(s.vdim) + s.eps) : 1.0f;
    const uint32_t pos = (a.pos0 + t) % s.capacity;
    T *blk = static_cast<T *>(a.v_cache) + (size_t(g) * (s.capacity / kKeyBlock) + pos / kKeyBlock) * s.dv_pad * kKeyBlock +
             value_slot<T>(pos % kKeyBlock);
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++) {
        const uint32_t d = lane + j * 64;
        if (d < s.vdim) blk[size_t(d) * kKeyBlock] = from_f32<T>(v[j] * r);
    }
}

// One head (blockIdx.x: q heads, then k, then v) of a run of tokens to a wave.
constexpr uint32_t kConvRun = 8;
__device__ __forceinline__ void conv_head_carry(const ConvCtx &x, const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t head) {
    const bool is_v = head >= s.heads + s.kv_heads;
    const uint32_t c0 = is_v ? (s.heads + s.kv_heads) * s.dim + (head - s.heads - s.kv_heads) * s.vdim : head * s.dim;
    for (uint32_t d = threadIdx.x; d < (is_v ? s.vdim : s.dim); d += 256) conv_carry(x, a.hist_out, a.n_tokens, c0 + d);
}

// any sizes: token by token
template <typename T>
__global__ __launch_bounds__(256) void conv_rotate_kernel(RmiAttnShape s, RmiAttnArgs a) {
    const uint32_t lane = threadIdx.x & 63, head = blockIdx.x;
    const uint32_t channels = (s.heads + s.kv_heads) * s.dim + s.kv_heads * s.vdim;
    const ConvCtx x{a.u, a.hist_in, a.conv, channels, s.taps};
    if (blockIdx.y == 0) conv_head_carry(x, s, a, head);  // one workgroup of a head also carries its history on
    const uint32_t t0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * kConvRun;
    for (uint32_t t = t0; t < t0 + kConvRun && t < a.n_tokens; t++) {
        if (head >= s.heads + s.kv_heads) {
            value_row<T>(x, s, a, t, head - s.heads - s.kv_heads, lane);
        } else if (head >= s.heads) {
            key_row<T>(x, s, a, t, head - s.heads, lane);
        } else {
            const uint32_t group = s.heads / s.kv_heads, g = head / group, r = head % group;
            T *row = static_cast<T *>(a.q) + (size_t(g) * a.n_tokens * group + size_t(t) * group + r) * s.dk_pad;
            for (uint32_t i = lane; i < s.dk_pad / 2; i += 64) {
                float p, q;
                conv_rotate_pair(x, s, a.cos_t, a.sin_t, t, a.pos0, head * s.dim, i, p, q);
                store_pair(row + 2 * i, p, q);
            }
        }
    }
}

// Even head sizes up to 128 and up to four taps: a lane holds one pair of channels.
__host__ __device__ inline bool conv_pairs_fit(const RmiAttnShape &s) {
    return s.taps <= 4 && s.dim % 2 == 0 && s.vdim % 2 == 0 && s.dim <= 128 && s.vdim <= 128;
}
// taps of channels c, c + 1, four each, the last one the token's own
struct PairTaps {
    float w0[4], w1[4];
    __device__ __forceinline__ void load(const RmiAttnShape &s, const float *conv, uint32_t c) {
        const uint32_t off = 4 - s.taps;
#pragma unroll
        for (uint32_t j = 0; j < 4; j++) {
            w0[j] = j >= off ? conv[c * s.taps + j - off] : 0.0f;
            w1[j] = j >= off ? conv[(c + 1) * s.taps + j - off] : 0.0f;
        }
    }
};
// the projected pair at the pass's row t - back (back <= 3); a position below zero reads as zero
__device__ __forceinline__ float2 pair_row(const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t channels, uint32_t t, uint32_t back, uint32_t c) {
    if (t >= back) return *reinterpret_cast<const float2 *>(a.u + size_t(t - back) * channels + c);
    if (back - t < s.taps && a.pos0 + t >= back) return *reinterpret_cast<const float2 *>(a.hist_in + size_t(t + s.taps - 1 - back) * channels + c);
    return make_float2(0.f, 0.f);
}

// A run of tokens: the taps and a sliding window of projected values stay in registers; every row is read once.
template <typename T>
__global__ __launch_bounds__(256) void conv_rotate_pairs_kernel(RmiAttnShape s, RmiAttnArgs a) {
    const uint32_t lane = threadIdx.x & 63, head = blockIdx.x;
    const uint32_t channels = (s.heads + s.kv_heads) * s.dim + s.kv_heads * s.vdim;
    const ConvCtx x{a.u, a.hist_in, a.conv, channels, s.taps};
    if (blockIdx.y == 0) conv_head_carry(x, s, a, head);
    // runs end at multiples of kConvRun positions: a value block takes four keys of a channel in one store
    const uint32_t p_run = a.pos0 / kConvRun * kConvRun + (blockIdx.y * 4 + uint32_t(__builtin_amdgcn_readfirstlane(int(threadIdx.x >> 6)))) * kConvRun;
    if (p_run >= a.pos0 + a.n_tokens) return;
    const uint32_t skip = p_run < a.pos0 ? a.pos0 - p_run : 0;  // positions of the first run that came before
    const uint32_t t0 = p_run + skip - a.pos0;
    const bool is_v = head >= s.heads + s.kv_heads, is_q = head < s.heads;
    const uint32_t dim = is_v ? s.vdim : s.dim;
    const uint32_t c0 = is_v ? (s.heads + s.kv_heads) * s.dim + (head - s.heads - s.kv_heads) * s.vdim : head * s.dim;
    const bool has = 2 * lane < dim;
    const uint32_t c = c0 + (has ? 2 * lane : 0);
    float u0[4], u1[4];  // row j of four, the last one the token's own
    PairTaps w;
    w.load(s, a.conv, c);
    float2 row[kConvRun];
#pragma unroll
    for (uint32_t i = 0; i < kConvRun; i++) {
        const uint32_t ti = i < skip ? 0 : p_run + i - a.pos0, t = ti < a.n_tokens ? ti : a.n_tokens - 1;
        row[i] = *reinterpret_cast<const float2 *>(a.u + size_t(t) * channels + c);
    }
#pragma unroll
    for (uint32_t j = 1; j < 4; j++) {  // the rows before the run
        const float2 v = pair_row(s, a, channels, t0, 4 - j, c);
        u0[j] = v.x;
        u1[j] = v.y;
    }
    const uint32_t group = s.heads / s.kv_heads, half = s.rot_dims / 2;
    const bool turned = !is_v && lane < half;
    T *out;  // of the first live token; `step` further for the next
    size_t step;
    if (is_q) {
        out = static_cast<T *>(a.q) + (size_t(head / group) * a.n_tokens * group + size_t(t0) * group + head % group) * s.dk_pad;
        step = size_t(group) * s.dk_pad;
    } else {
        out = static_cast<T *>(a.k_cache) + (size_t(head - s.heads) * s.capacity + (a.pos0 + t0) % s.capacity) * s.dk_pad;  // (a run does not wrap)
        step = s.dk_pad;
    }
    float v0[kConvRun], v1[kConvRun];
    uint32_t n_live = skip;  // one past the last live place of the run
#pragma unroll
    for (uint32_t i = 0; i < kConvRun; i++) {
        v0[i] = v1[i] = 0.0f;
        if (i < skip || p_run + i >= a.pos0 + a.n_tokens) continue;
        n_live = i + 1;
#pragma unroll
        for (uint32_t j = 0; j < 3; j++) {
            u0[j] = u0[j + 1];
            u1[j] = u1[j + 1];
        }
        u0[3] = row[i].x;
        u1[3] = row[i].y;
        float p = 0.0f, q = 0.0f;
#pragma unroll
        for (uint32_t j = 0; j < 4; j++) {
            p = __builtin_fmaf(w.w0[j], u0[j], p);
            q = __builtin_fmaf(w.w1[j], u1[j], q);
        }
        if (!has) p = q = 0.0f;
        if (is_v) {
            const float r = s.v_norm ? 1.0f / sqrtf(wave_sum_f32(__builtin_fmaf(p, p, q * q)) / float(dim) + s.eps) : 1.0f;
            v0[i] = p * r;
            v1[i] = q * r;
        } else {
            if (turned) {
                const size_t at = size_t(p_run + i) * half + lane;
                const float cs = a.cos_t[at], sn = a.sin_t[at], rp = p;
                p = __builtin_fmaf(rp, cs, -(q * sn));
                q = __builtin_fmaf(q, cs, rp * sn);
            }
            if (2 * lane < s.dk_pad) store_pair(out + (i - skip) * step + 2 * lane, p, q);
        }
    }
    if (is_v && has) {
        T *blk = static_cast<T *>(a.v_cache) +
                 (size_t(head - s.heads - s.kv_heads) * (s.capacity / kKeyBlock) + p_run % s.capacity / kKeyBlock) * s.dv_pad * kKeyBlock +
                 size_t(2 * lane) * kKeyBlock;
#pragma unroll
        for (uint32_t g = 0; g < kConvRun; g += 4) {  // four keys lie side by side
            T *dst = blk + value_slot<T>((p_run + g) % kKeyBlock);
            if (g >= skip && g + 4 <= n_live) {
                store4(dst, f32x4{v0[g], v0[g + 1], v0[g + 2], v0[g + 3]});
                store4(dst + kKeyBlock, f32x4{v1[g], v1[g + 1], v1[g + 2], v1[g + 3]});
            } else {
#pragma unroll
                for (uint32_t i = g; i < g + 4; i++)
                    if (i >= skip && i < n_live) {
                        dst[i - g] = from_f32<T>(v0[i]);
                        dst[kKeyBlock + i - g] = from_f32<T>(v1[i]);
                    }
            }
        }
    }
}

// ---- attention.  The columns of a key/value head are its pass's (token, query head of the group) pairs, token by
// token; a wave takes QT tiles of sixteen.  Scores come as K q (rows: keys, columns: queries), so a lane holds the
// weights of one column and the running maximum and sum are a lane's own; the weights then are the operand of
// V^T p as they lie, because the value blocks hold their keys in that order.
template <typename T, int BUCKET, int QT>
struct AttnWave {
    static constexpr uint32_t kKC = BUCKET / (4 * kPieceElems<T>);  // 16-byte pieces a lane holds of a head's keys
    static constexpr uint32_t kVT = BUCKET / 16;
    f32x4 o[QT][kVT];
    float m[QT], l[QT];
    u32x4 qf[QT][kKC];

    __device__ __forceinline__ void init() {
#pragma unroll
        for (int i = 0; i < QT; i++) {
            m[i] = -INFINITY;
            l[i] = 0.0f;
#pragma unroll
            for (uint32_t v = 0; v < kVT; v++) o[i][v] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
    }
    // a block's keys and values fit in registers beside the rest: values of a block and keys of the next are under way
    // while the block's scores and weights are computed
    static constexpr bool kAhead = BUCKET * sizeof(T) <= 256;
    u32x4 kf[2][kAhead ? kKC : 1], vf[kAhead ? kVT * (sizeof(T) / 2) : 1];

    __device__ __forceinline__ void load_keys(const T *kc, const RmiAttnShape &s, uint32_t k) {
        const uint32_t lane = threadIdx.x & 63, n_kc = s.dk_pad / (4 * kPieceElems<T>);
        const T *row = kc + size_t(k + (lane & 15)) * s.dk_pad + (lane >> 4) * kPieceElems<T>;
#pragma unroll
        for (uint32_t c = 0; c < (kAhead ? kKC : 0); c++) {
            if (c >= n_kc) continue;
            kf[0][c] = *reinterpret_cast<const u32x4 *>(row + c * 4 * kPieceElems<T>);
            kf[1][c] = *reinterpret_cast<const u32x4 *>(row + c * 4 * kPieceElems<T> + 16 * size_t(s.dk_pad));
        }
    }
    __device__ __forceinline__ const T *value_at(const T *vc, const RmiAttnShape &s, uint32_t k) {
        const uint32_t lane = threadIdx.x & 63;
        return vc + size_t(k / kKeyBlock) * s.dv_pad * kKeyBlock + size_t(lane & 15) * kKeyBlock + (lane >> 4) * kPieceElems<T>;
    }
    __device__ __forceinline__ void load_values(const T *vc, const RmiAttnShape &s, uint32_t k) {
        const T *vb = value_at(vc, s, k);
        const uint32_t n_vt = s.dv_pad / 16;
#pragma unroll
        for (uint32_t v = 0; v < (kAhead ? kVT : 0); v++)
#pragma unroll
            for (uint32_t t = 0; t < sizeof(T) / 2; t++)
                if (v < n_vt) vf[v * (sizeof(T) / 2) + t] = *reinterpret_cast<const u32x4 *>(vb + size_t(v) * 16 * kKeyBlock + t * 16);
    }
    // keys [k0, k1), k0 a multiple of 32; column i sees keys up to last[i] (< k1 not required) and, with a window, from
    // last[i] - window + 1 on.  loaded: the first block's keys and values are in kf and vf
    __device__ __forceinline__ void keys(const T *kc, const T *vc, const RmiAttnShape &s, uint32_t k0, uint32_t k1, const int (&last)[QT],
                                         bool loaded = false) {
        const uint32_t lane = threadIdx.x & 63, fr = lane & 15, g = lane >> 4;
        const uint32_t n_kc = s.dk_pad / (4 * kPieceElems<T>), n_vt = s.dv_pad / 16;
        const T *krow = kc + size_t(fr) * s.dk_pad + g * kPieceElems<T>;
        uint32_t row = k0 % s.capacity;  // where the block lies
        if (!loaded && k0 < k1) load_keys(kc, s, row);
        for (uint32_t k = k0; k < k1; k += kKeyBlock) {
            const T *vb = value_at(vc, s, row);
            if (!loaded || k != k0) load_values(vc, s, row);
            const uint32_t next = row + kKeyBlock < s.capacity ? row + kKeyBlock : 0;
            f32x4 sc[QT][2];
#pragma unroll
            for (int i = 0; i < QT; i++) sc[i][0] = sc[i][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (uint32_t c = 0; c < kKC; c++) {
                if (c >= n_kc) continue;
                u32x4 f0, f1;
                if constexpr (kAhead) {
                    f0 = kf[0][c];
                    f1 = kf[1][c];
                } else {
                    const T *p = krow + size_t(row) * s.dk_pad + c * 4 * kPieceElems<T>;
                    f0 = *reinterpret_cast<const u32x4 *>(p);
                    f1 = *reinterpret_cast<const u32x4 *>(p + 16 * size_t(s.dk_pad));
                }
#pragma unroll
                for (int i = 0; i < QT; i++) {
                    sc[i][0] = mma16<T>(f0, qf[i][c], sc[i][0]);
                    sc[i][1] = mma16<T>(f1, qf[i][c], sc[i][1]);
                }
            }
            if (k + kKeyBlock < k1) load_keys(kc, s, next);
            row = next;
            u32x4 pf[QT][2];
#pragma unroll
            for (int i = 0; i < QT; i++) {
                float top = -INFINITY;
                const int first = s.window ? last[i] - int(s.window) + 1 : 0;
#pragma unroll
                for (int t = 0; t < 2; t++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int key = int(k) + t * 16 + int(g) * 4 + r;
                        sc[i][t][r] = key >= first && key <= last[i] && key < int(k1) ? sc[i][t][r] * s.scale : -INFINITY;
                        top = fmaxf(top, sc[i][t][r]);
                    }
                const float m_new = fmaxf(m[i], rows_max_f32(top));
                const float ref = m_new == -INFINITY ? 0.0f : m_new;  // nothing visible yet: every weight stays zero
                const float keep = exp_t<T>(m[i] - ref);
                float sum = 0.0f;
#pragma unroll
                for (int t = 0; t < 2; t++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        sc[i][t][r] = exp_t<T>(sc[i][t][r] - ref);
                        sum += sc[i][t][r];
                    }
                m[i] = m_new;
                l[i] = __builtin_fmaf(l[i], keep, sum);
#pragma unroll
                for (uint32_t v = 0; v < kVT; v++) o[i][v] *= keep;
                if constexpr (sizeof(T) == 2) {
                    bf16x8 b;
#pragma unroll
                    for (int r = 0; r < 8; r++) b[r] = static_cast<__bf16>(sc[i][r >> 2][r & 3]);
                    pf[i][0] = __builtin_bit_cast(u32x4, b);
                } else {
                    pf[i][0] = __builtin_bit_cast(u32x4, sc[i][0]);
                    pf[i][1] = __builtin_bit_cast(u32x4, sc[i][1]);
                }
            }
#pragma unroll
            for (uint32_t v = 0; v < kVT; v++) {
                if (v >= n_vt) continue;
#pragma unroll
                for (uint32_t t = 0; t < sizeof(T) / 2; t++) {
                    const u32x4 f = kAhead ? vf[kAhead ? v * (sizeof(T) / 2) + t : 0]
                                           : *reinterpret_cast<const u32x4 *>(vb + size_t(v) * 16 * kKeyBlock + t * 16);
#pragma unroll
                    for (int i = 0; i < QT; i++) o[i][v] = mma16<T>(f, pf[i][t], o[i][v]);
                }
            }
        }
    }
};

// the block in which the first key lies that position p sees
__device__ __forceinline__ uint32_t first_block(const RmiAttnShape &s, uint32_t p) {
    return s.window && p + 1 > s.window ? (p + 1 - s.window) / kKeyBlock * kKeyBlock : 0;
}

// four channels d .. d + 3 of a finished column
template <typename T>
__device__ __forceinline__ void attn_store(const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t t, uint32_t head, uint32_t d, f32x4 v) {
    T *dst = static_cast<T *>(a.out) + size_t(t) * a.out_ld + size_t(head) * s.vdim + d;
    if (d + 3 < s.vdim && (s.vdim & 3) == 0) {  // out_ld is a multiple of 64
        store4(dst, v);
    } else {
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (d + r < s.vdim) dst[r] = from_f32<T>(v[r]);
    }
}

// several tokens: a workgroup takes QT tiles, each of its four waves a quarter of the keys they see; merged in LDS
template <typename T, int BUCKET, int QT>
__global__ __launch_bounds__(256) void attn_pass_kernel(RmiAttnShape s, RmiAttnArgs a) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), fr = lane & 15, g4 = lane >> 4;
    const uint32_t group = s.heads / s.kv_heads, kvh = blockIdx.x % s.kv_heads, n_cols = a.n_tokens * group;
    const uint32_t tile = gridDim.x / s.kv_heads - 1 - blockIdx.x / s.kv_heads;  // the longest columns first
    AttnWave<T, BUCKET, QT> w;
    w.init();
    int last[QT];
    const uint32_t n_kc = s.dk_pad / (4 * kPieceElems<T>);
#pragma unroll
    for (int i = 0; i < QT; i++) {
        const uint32_t col = (tile * QT + i) * 16 + fr, cc = col < n_cols ? col : n_cols - 1;
        last[i] = int(a.pos0 + cc / group);
        const T *q = static_cast<const T *>(a.q) + (size_t(kvh) * n_cols + cc) * s.dk_pad + g4 * kPieceElems<T>;
#pragma unroll
        for (uint32_t c = 0; c < w.kKC; c++) {
            if (c >= n_kc) continue;
            w.qf[i][c] = *reinterpret_cast<const u32x4 *>(q + c * 4 * kPieceElems<T>);
        }
    }
    const uint32_t first_col = tile * QT * 16, live = n_cols - first_col < QT * 16 ? n_cols - first_col : QT * 16;
    const uint32_t n_keys = a.pos0 + (first_col + live - 1) / group + 1, begin = first_block(s, a.pos0 + first_col / group);
    const uint32_t per_wave = (n_keys - begin + 4 * kKeyBlock - 1) / (4 * kKeyBlock) * kKeyBlock;
    const uint32_t k0 = begin + wave * per_wave, k1 = k0 + per_wave < n_keys ? k0 + per_wave : n_keys;
    if (k0 < k1)
        w.keys(static_cast<const T *>(a.k_cache) + size_t(kvh) * s.capacity * s.dk_pad,
               static_cast<const T *>(a.v_cache) + size_t(kvh) * s.capacity * s.dv_pad, s, k0, k1, last);
    // [wave][maxima, sums, column x channel (rows a float4 apart more than they hold)]
    const uint32_t row = s.dv_pad + 4, pl = QT * 16 * (row + 2);
    float *all = reinterpret_cast<float *>(lds_raw), *mine = all + wave * pl;
#pragma unroll
    for (int i = 0; i < QT; i++) {
        const float l = rows_sum_f32(w.l[i]);
        if (g4 == 0) {
            mine[i * 16 + fr] = w.m[i];
            mine[QT * 16 + i * 16 + fr] = l;
        }
#pragma unroll
        for (uint32_t v = 0; v < w.kVT; v++)
            if (v * 16 < s.dv_pad) *reinterpret_cast<f32x4 *>(mine + QT * 32 + (i * 16 + fr) * row + v * 16 + g4 * 4) = w.o[i][v];
    }
    __syncthreads();
    const uint32_t quads = s.dv_pad / 4;
    for (uint32_t e = tid; e < live * quads; e += 256) {
        const uint32_t c = e / quads, d = e % quads * 4;
        float m = all[c];
#pragma unroll
        for (uint32_t i = 1; i < 4; i++) m = fmaxf(m, all[i * pl + c]);
        float sum = 0.0f;  // (every column sees its own key: m is finite)
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (uint32_t i = 0; i < 4; i++) {
            const float f = exp_t<T>(all[i * pl + c] - m);
            sum = __builtin_fmaf(all[i * pl + QT * 16 + c], f, sum);
            o += *reinterpret_cast<const f32x4 *>(all + i * pl + QT * 32 + c * row + d) * f;
        }
        const uint32_t mc = first_col + c, t = mc / group, head = kvh * group + mc % group;
        attn_store<T>(s, a, t, head, d, o * ((a.gate ? a.gate[size_t(t) * s.heads + head] : 1.0f) / sum));
    }
}

// Few columns: the keys are divided over `parts` workgroups and their four waves; each workgroup merges its waves in
// LDS, writes its part, and the one that arrives last merges the parts.  With one token (STEP) the workgroup makes
// its queries itself, and the workgroups of the last part the new key and value.
constexpr uint32_t kMaxParts = 32;
constexpr uint32_t kStepThreads = 256;  // a workgroup of the single-token launch
// a part: the columns' maxima, their sums, and [column][channel]
__host__ __device__ inline uint32_t attn_part_floats(uint32_t dv_pad) { return 16 * (dv_pad + 2); }

template <typename T, int BUCKET, bool STEP>
__device__ __forceinline__ void attn_split(const RmiAttnShape &s, const RmiAttnArgs &a, uint32_t block, uint32_t parts, uint32_t keys_per_part,
                                           uint8_t *lds, uint32_t *flag) {
    constexpr uint32_t NW = 4;
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), fr = lane & 15, g4 = lane >> 4;
    const uint32_t group = s.heads / s.kv_heads, n_cols = a.n_tokens * group, tiles = (n_cols + 15) / 16;
    const uint32_t part = block % parts, ct = (block / parts) % tiles, kvh = block / parts / tiles;
    const uint32_t last_col = ct * 16 + 15 < n_cols ? ct * 16 + 15 : n_cols - 1;
    const uint32_t begin = first_block(s, a.pos0 + ct * 16 / group), n_keys = a.pos0 + last_col / group + 1;  // what the tile sees
    const uint32_t n_kc = s.dk_pad / (4 * kPieceElems<T>);
    AttnWave<T, BUCKET, 1> w;
    w.init();
    const uint32_t col = ct * 16 + fr, cc = col < n_cols ? col : n_cols - 1;
    const int last[1] = {int(a.pos0 + cc / group)};
    const T *kc = static_cast<const T *>(a.k_cache) + size_t(kvh) * s.capacity * s.dk_pad;
    const T *vc = static_cast<const T *>(a.v_cache) + size_t(kvh) * s.capacity * s.dv_pad;
    const uint32_t p0 = begin + part * keys_per_part, p1 = p0 + keys_per_part < n_keys ? p0 + keys_per_part : n_keys;
    const uint32_t per_wave = keys_per_part / NW;  // a multiple of the key block
    const uint32_t k0 = p0 + wave * per_wave, k1 = k0 + per_wave < p1 ? k0 + per_wave : p1;
    bool loaded = false;
    if constexpr (STEP) {
        T *q = reinterpret_cast<T *>(lds);
        const uint32_t channels = (s.heads + s.kv_heads) * s.dim + s.kv_heads * s.vdim;
        const ConvCtx x{a.u, a.hist_in, a.conv, channels, s.taps};
        const uint32_t half = s.dk_pad / 2, c_end = n_cols - ct * 16 < 16 ? n_cols - ct * 16 : 16;
        const uint32_t own = a.pos0 % s.capacity;
        const bool newest = a.pos0 - p0 < keys_per_part;  // this part holds the token's own key and value
        // the first block of keys and values: under way behind the convolution's operands, unless it holds the new one
        auto ahead = [&] {
            loaded = w.kAhead && k0 < k1 && k0 + kKeyBlock < n_keys;
            if (loaded) {
                w.load_keys(kc, s, k0 % s.capacity);
                w.load_values(vc, s, k0 % s.capacity);
            }
        };
        if (conv_pairs_fit(s)) {
            // with the new key and value to make, the last two waves make them and the others the queries
            const uint32_t q_threads = newest ? 128 : 256, rot = s.rot_dims / 2;
            const bool is_k = newest && wave == 2, is_v = newest && wave == 3;
            const uint32_t n_pairs = is_v ? s.vdim / 2 : is_k ? half : c_end * half, step = is_k || is_v ? 64 : q_threads;
            bool first = true;
            for (uint32_t e0 = 0; e0 < n_pairs || first; e0 += step) {
                const uint32_t e = e0 + (is_k || is_v ? lane : tid), ec = e < n_pairs ? e : 0;
                const uint32_t c = is_k || is_v ? 0 : ec / half, i = is_k || is_v ? ec : ec % half;
                const bool has = e < n_pairs && (is_v || 2 * i < s.dim);
                const uint32_t c0 = is_v   ? (s.heads + s.kv_heads) * s.dim + kvh * s.vdim
                                    : is_k ? (s.heads + kvh) * s.dim
                                           : (kvh * group + ct * 16 + c) * s.dim;
                const uint32_t ch = c0 + (has ? 2 * i : 0);
                PairTaps t;
                float2 r[4];
#pragma unroll
                for (uint32_t j = 0; j < 4; j++) r[j] = pair_row(s, a, channels, 0, 3 - j, ch);
                t.load(s, a.conv, ch);
                const bool turned = has && !is_v && i < rot;
                const size_t at = size_t(a.pos0) * rot + (turned ? i : 0);
                const float cs = turned ? a.cos_t[at] : 1.0f, sn = turned ? a.sin_t[at] : 0.0f;
                if (first) ahead();
                first = false;
                float p = 0.0f, o = 0.0f;
#pragma unroll
                for (uint32_t j = 0; j < 4; j++) {
                    p = __builtin_fmaf(t.w0[j], r[j].x, p);
                    o = __builtin_fmaf(t.w1[j], r[j].y, o);
                }
                if (!has) p = o = 0.0f;
                if (is_v) {  // (at most 64 pairs: one round)
                    const float f = s.v_norm ? 1.0f / sqrtf(wave_sum_f32(__builtin_fmaf(p, p, o * o)) / float(s.vdim) + s.eps) : 1.0f;
                    T *blk = const_cast<T *>(vc) + size_t(own / kKeyBlock) * s.dv_pad * kKeyBlock + value_slot<T>(own % kKeyBlock);
                    if (has) {
                        blk[size_t(2 * i) * kKeyBlock] = from_f32<T>(p * f);
                        blk[size_t(2 * i + 1) * kKeyBlock] = from_f32<T>(o * f);
                    }
                } else if (e < n_pairs) {
                    const float rp = p;
                    p = __builtin_fmaf(rp, cs, -(o * sn));
                    o = __builtin_fmaf(o, cs, rp * sn);
                    store_pair(is_k ? const_cast<T *>(kc) + size_t(own) * s.dk_pad + 2 * i : q + c * s.dk_pad + 2 * i, p, o);
                }
            }
        } else {
            if (newest) {
                if (wave == NW - 2) key_row<T>(x, s, a, 0, kvh, lane);
                if (wave == NW - 1) value_row<T>(x, s, a, 0, kvh, lane);
            }
            for (uint32_t e = tid; e < c_end * half; e += 256) {
                const uint32_t c = e / half, i = e % half, head = kvh * group + ct * 16 + c;
                float p, r;
                conv_rotate_pair(x, s, a.cos_t, a.sin_t, 0, a.pos0, head * s.dim, i, p, r);
                store_pair(q + c * s.dk_pad + 2 * i, p, r);
            }
        }
        __syncthreads();
        const uint32_t qc = fr < c_end ? fr : c_end - 1;
#pragma unroll
        for (uint32_t c = 0; c < w.kKC; c++) {
            if (c >= n_kc) continue;
            w.qf[0][c] = *reinterpret_cast<const u32x4 *>(q + qc * s.dk_pad + (c * 4 + g4) * kPieceElems<T>);
        }
        __syncthreads();
    } else {
        const T *q = static_cast<const T *>(a.q) + (size_t(kvh) * n_cols + cc) * s.dk_pad + g4 * kPieceElems<T>;
#pragma unroll
        for (uint32_t c = 0; c < w.kKC; c++) {
            if (c >= n_kc) continue;
            w.qf[0][c] = *reinterpret_cast<const u32x4 *>(q + c * 4 * kPieceElems<T>);
        }
    }
    if (k0 < k1) w.keys(kc, vc, s, k0, k1, last, loaded);
    if constexpr (STEP) {
        if (part == 0) {  // the history of this workgroup's channels
            const uint32_t channels = (s.heads + s.kv_heads) * s.dim + s.kv_heads * s.vdim;
            const ConvCtx x{a.u, a.hist_in, a.conv, channels, s.taps};
            const uint32_t c_end = n_cols - ct * 16 < 16 ? n_cols - ct * 16 : 16, c0 = (kvh * group + ct * 16) * s.dim;
            for (uint32_t d = tid; d < c_end * s.dim; d += 256) conv_carry(x, a.hist_out, 1, c0 + d);
            if (ct == 0) {
                for (uint32_t d = tid; d < s.dim; d += 256) conv_carry(x, a.hist_out, 1, (s.heads + kvh) * s.dim + d);
                for (uint32_t d = tid; d < s.vdim; d += 256)
                    conv_carry(x, a.hist_out, 1, (s.heads + s.kv_heads) * s.dim + kvh * s.vdim + d);
            }
        }
    }
    // the waves' results to LDS, live columns only; then every thread merges (column, channel) pairs
    const uint32_t live = n_cols - ct * 16 < 16 ? n_cols - ct * 16 : 16, pf = attn_part_floats(s.dv_pad), pl = 32 + live * s.dv_pad;
    float *all = reinterpret_cast<float *>(lds), *mine = all + wave * pl;
    const float l = rows_sum_f32(w.l[0]);
    if (fr < live) {
        if (g4 == 0) {
            mine[fr] = w.m[0];
            mine[16 + fr] = l;
        }
#pragma unroll
        for (uint32_t v = 0; v < w.kVT; v++)
            if (v * 16 < s.dv_pad) *reinterpret_cast<f32x4 *>(mine + 32 + fr * s.dv_pad + v * 16 + g4 * 4) = w.o[0][v];
    }
    __syncthreads();
    const uint32_t slot = kvh * tiles + ct;
    float *ws = reinterpret_cast<float *>(static_cast<uint32_t *>(a.scratch) + kAttnCounters) + size_t(slot) * parts * pf;
    const uint32_t pairs = live * s.dv_pad;
    auto finish = [&](uint32_t e, float o, float sum) {
        const uint32_t c = e / s.dv_pad, d = e % s.dv_pad;
        if (d >= s.vdim) return;
        const uint32_t mc = ct * 16 + c, t = mc / group, head = kvh * group + mc % group;
        static_cast<T *>(a.out)[size_t(t) * a.out_ld + size_t(head) * s.vdim + d] =
            from_f32<T>(o * ((a.gate ? a.gate[size_t(t) * s.heads + head] : 1.0f) / sum));
    };
    for (uint32_t e = tid; e < pairs; e += 256) {
        const uint32_t c = e / s.dv_pad;
        float m = all[c];
#pragma unroll
        for (uint32_t i = 1; i < NW; i++) m = fmaxf(m, all[i * pl + c]);
        const float ref = m == -INFINITY ? 0.0f : m;  // a column that sees no key of this part
        float sum = 0.0f, o = 0.0f;
#pragma unroll
        for (uint32_t i = 0; i < NW; i++) {
            const float f = exp_t<T>(all[i * pl + c] - ref);
            sum = __builtin_fmaf(all[i * pl + 16 + c], f, sum);
            o = __builtin_fmaf(all[i * pl + 32 + e], f, o);
        }
        if (parts == 1) {
            finish(e, o, sum);
        } else {
            float *dst = ws + size_t(part) * pf;
            if (e % s.dv_pad == 0) {
                __hip_atomic_store(dst + c, m, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                __hip_atomic_store(dst + 16 + c, sum, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
            __hip_atomic_store(dst + 32 + e, o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
    }
    if (parts == 1) return;
    // Hand-over between workgroups.  Everything handed over is written and read by agent-scope atomics, past the caches
    // that are not coherent; a wave's stores are complete before it arrives at the barrier, and the workgroup counts
    // behind the barrier, so no cache has to be written back or invalidated.
    __builtin_amdgcn_s_waitcnt(0);
    __syncthreads();
    if (tid == 0) {
        uint32_t *count = static_cast<uint32_t *>(a.scratch) + slot;
        const uint32_t n = __hip_atomic_fetch_add(count, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        *flag = n == parts - 1;
        if (n == parts - 1) __hip_atomic_store(count, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);  // ready for the next launch
    }
    __syncthreads();
    if (!*flag) return;
    for (uint32_t e = tid; e < pairs; e += 256) {
        const uint32_t c = e / s.dv_pad;
        float m = -INFINITY, sum = 0.0f, o = 0.0f;
        for (uint32_t p0 = 0; p0 < parts; p0 += 8) {  // eight parts' loads at a time
            float mv[8], lv[8], ov[8];
#pragma unroll
            for (uint32_t j = 0; j < 8; j++) {
                const float *src = ws + size_t(p0 + j < parts ? p0 + j : parts - 1) * pf;
                mv[j] = __hip_atomic_load(src + c, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                lv[j] = __hip_atomic_load(src + 16 + c, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                ov[j] = __hip_atomic_load(src + 32 + e, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
            float top = m;
#pragma unroll
            for (uint32_t j = 0; j < 8; j++)
                if (p0 + j < parts) top = fmaxf(top, mv[j]);
            const float ref = top == -INFINITY ? 0.0f : top, keep = exp_t<T>(m - ref);
            sum *= keep;
            o *= keep;
#pragma unroll
            for (uint32_t j = 0; j < 8; j++) {
                const float f = p0 + j < parts ? exp_t<T>(mv[j] - ref) : 0.0f;
                sum = __builtin_fmaf(lv[j], f, sum);
                o = __builtin_fmaf(ov[j], f, o);
            }
            m = top;
        }
        finish(e, o, sum);
    }
}

template <typename T, int BUCKET>
__global__ __launch_bounds__(256) void attn_split_kernel(RmiAttnShape s, RmiAttnArgs a, uint32_t parts, uint32_t keys_per_part) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    __shared__ uint32_t flag;
    attn_split<T, BUCKET, false>(s, a, blockIdx.x, parts, keys_per_part, lds_raw, &flag);
}

// ---- gated linear recurrence
// one token of one head: a thread takes four state columns and every (kStepThreads / (v_pad / 4))-th row
template <typename T>
__device__ __forceinline__ void recur_step(const RmiRecurShape &s, const RmiRecurArgs &a, uint32_t head, float *lds) {
    const uint32_t tid = threadIdx.x, quads = s.v_pad / 4, slices = kStepThreads / quads;
    float *fs = lds, *qs = fs + s.d_pad, *vs = qs + s.d_pad, *part = vs + s.v_pad;  // part [slices][v_pad]
    for (uint32_t d = tid; d < s.d_pad; d += kStepThreads) {
        fs[d] = d < s.dim ? a.f[head * s.dim + d] : 1.0f;
        qs[d] = d < s.dim ? a.q[head * s.dim + d] : 0.0f;
    }
    for (uint32_t d = tid; d < s.v_pad; d += kStepThreads) vs[d] = d < s.vdim ? a.v[head * s.vdim + d] : 0.0f;
    __syncthreads();
    const uint32_t c = tid % quads, sl = tid / quads;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    if (sl < slices) {
        const size_t at = size_t(head) * s.d_pad * s.v_pad + c * 4;
        const float *st = a.state_in + at;
        float *st_out = a.state_out + at;
        const f32x4 v = *reinterpret_cast<const f32x4 *>(vs + c * 4);
        for (uint32_t d0 = sl; d0 < s.d_pad; d0 += slices * 8) {  // eight rows in flight
            f32x4 r[8];
#pragma unroll
            for (uint32_t j = 0; j < 8; j++) {
                const uint32_t d = d0 + j * slices;
                r[j] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (a.pos0 && d < s.d_pad) r[j] = *reinterpret_cast<const f32x4 *>(st + size_t(d) * s.v_pad);
            }
#pragma unroll
            for (uint32_t j = 0; j < 8; j++) {
                const uint32_t d = d0 + j * slices;
                if (d >= s.d_pad) break;
                const float f = fs[d], k = 1.0f - f, q = qs[d];
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    r[j][e] = __builtin_fmaf(f, r[j][e], k * v[e]);
                    o[e] = __builtin_fmaf(q, r[j][e], o[e]);
                }
                *reinterpret_cast<f32x4 *>(st_out + size_t(d) * s.v_pad) = r[j];
            }
        }
        *reinterpret_cast<f32x4 *>(part + sl * s.v_pad + c * 4) = o;
    }
    __syncthreads();
    float *red = fs;  // fs is read no more
    float mine = 0.0f;
    if (tid < s.vdim)
        for (uint32_t i = 0; i < slices; i++) mine += part[i * s.v_pad + tid];
    const float sq = wave_sum_f32(mine * mine);
    if ((tid & 63) == 0) red[tid >> 6] = sq;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (uint32_t i = 0; i < kStepThreads / 64; i++) total += red[i];
    const float r = 1.0f / sqrtf(total / float(s.vdim) + s.eps);
    if (tid < s.vdim) static_cast<T *>(a.out)[size_t(head) * s.vdim + tid] = from_f32<T>(mine * r * a.norm[tid]);
}
inline size_t recur_step_lds(const RmiRecurShape &s) {
    return (2 * size_t(s.d_pad) + s.v_pad + size_t(kStepThreads / (s.v_pad / 4)) * s.v_pad) * 4;
}

template <typename T, int BUCKET>
__global__ __launch_bounds__(kStepThreads) void mixers_step_kernel(RmiAttnShape s, RmiAttnArgs a, uint32_t attn_blocks, uint32_t parts,
                                                          uint32_t keys_per_part, RmiRecurShape rs, RmiRecurArgs ra) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    __shared__ uint32_t flag;
    if (blockIdx.x < attn_blocks)
        attn_split<T, BUCKET, true>(s, a, blockIdx.x, parts, keys_per_part, lds_raw, &flag);
    else
        recur_step<T>(rs, ra, blockIdx.x - attn_blocks, reinterpret_cast<float *>(lds_raw));
}

// Several tokens, in chunks of sixteen.  With P_t the product of f over the chunk's tokens up to t:
//   o_t = (q_t P_t) S_0 + sum_{s <= t} A_ts v_s,   A_ts = sum_d q_t (1 - f_s) f_{s+1} .. f_t
//   S'  = P_15 S_0 + sum_s ((1 - f_s) f_{s+1} .. f_15) v_s
// Every factor is a product of forget gates, at most one: nothing is divided by a decay, so channels that forget
// at once are as exact as those that never do.  The first kernel makes the factors (all chunks at once), the
// second walks the chunks with the state in the matrix cores' accumulators.
constexpr uint32_t kChunk = 16;
constexpr uint32_t kMaxSegs = 8;
struct RecurScratch {
    float *qp, *kt, *am, *pc, *o, *seg_state, *seg_decay;
};
__host__ __device__ inline RecurScratch recur_scratch_at(float *p, const RmiRecurShape &s, uint32_t n_chunks) {
    const size_t hc = size_t(s.heads) * n_chunks;
    RecurScratch r;
    r.qp = p;                               // [head][chunk][16][d_pad]
    r.kt = r.qp + hc * kChunk * s.d_pad;    // [head][chunk][d_pad][16]
    r.am = r.kt + hc * kChunk * s.d_pad;    // [head][chunk][16 t][16 s]
    r.pc = r.am + hc * kChunk * kChunk;     // [head][chunk][d_pad]
    r.o = r.pc + hc * s.d_pad;              // [head][chunk][16][v_pad]
    r.seg_state = r.o + hc * kChunk * s.v_pad;  // [segment][head][d_pad][v_pad]
    r.seg_decay = r.seg_state + size_t(kMaxSegs) * s.heads * s.d_pad * s.v_pad;  // [segment][head][d_pad]
    return r;
}

// one chunk of one head
__global__ __launch_bounds__(256) void recur_factors_kernel(RmiRecurShape s, RmiRecurArgs a, uint32_t n_chunks) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    float *fl = reinterpret_cast<float *>(lds_raw);            // [16][d_pad + 4]
    const uint32_t ld = s.d_pad + 4;
    float *ql = fl + kChunk * ld;                              // [16][d_pad + 4]
    float *red = ql + kChunk * ld;                             // [4][16][16]
    const uint32_t tid = threadIdx.x, chunk = blockIdx.x, head = blockIdx.y, t0 = chunk * kChunk;
    const RecurScratch ws = recur_scratch_at(a.scratch, s, n_chunks);
    const size_t hc = size_t(head) * n_chunks + chunk;
    for (uint32_t e = tid; e < kChunk * s.d_pad; e += 256) {
        const uint32_t t = e / s.d_pad, d = e % s.d_pad;
        const bool live = t0 + t < a.n_tokens && d < s.dim;
        const size_t at = size_t(t0 + t) * s.heads * s.dim + size_t(head) * s.dim + d;
        fl[t * ld + d] = live ? a.f[at] : 1.0f;  // a token past the end changes nothing
        ql[t * ld + d] = live ? a.q[at] : 0.0f;
    }
    __syncthreads();
    for (uint32_t d = tid; d < s.d_pad; d += 256) {
        float p = 1.0f;
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            p *= fl[t * ld + d];
            ws.qp[(hc * kChunk + t) * s.d_pad + d] = ql[t * ld + d] * p;
        }
        ws.pc[hc * s.d_pad + d] = p;
        float k[kChunk];
        p = 1.0f;
#pragma unroll
        for (int t = kChunk - 1; t >= 0; t--) {
            const float f = fl[t * ld + d];
            k[t] = (1.0f - f) * p;
            p *= f;
        }
#pragma unroll
        for (uint32_t j = 0; j < kChunk / 4; j++)
            *reinterpret_cast<f32x4 *>(ws.kt + (hc * s.d_pad + d) * kChunk + 4 * j) = f32x4{k[4 * j], k[4 * j + 1], k[4 * j + 2], k[4 * j + 3]};
    }
    // A: thread (column s, slice of channels)
    const uint32_t col = tid & 15, slice = tid >> 4;
    float acc[kChunk];
#pragma unroll
    for (uint32_t t = 0; t < kChunk; t++) acc[t] = 0.0f;
    for (uint32_t d = slice; d < s.d_pad; d += 16) {
        float w = 0.0f;
        const float k = 1.0f - fl[col * ld + d];
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            w = t == col ? k : w * fl[t * ld + d];
            acc[t] = __builtin_fmaf(ql[t * ld + d], w, acc[t]);
        }
    }
#pragma unroll
    for (uint32_t t = 0; t < kChunk; t++) {
        const float v = rows_sum_f32(acc[t]);  // the wave's four slices
        if ((tid & 63) < 16) red[(tid >> 6) * 256 + t * 16 + col] = v;
    }
    __syncthreads();
    ws.am[hc * 256 + tid] = (red[tid] + red[256 + tid]) + (red[512 + tid] + red[768 + tid]);
}

// One workgroup: sixteen value channels of one head over the chunks of one segment of the pass; wave w holds the
// state's row tiles w, w + 4, ..  A tile of the state in accumulator form (row 4g + r in register r) is the right
// operand of (q P) S as it lies.  The segments of a long pass run side by side: a first launch (STATE_ONLY) takes every
// segment but the last from a zero state and leaves what it adds and how much it keeps; the second puts its starting
// state together from those before it.
template <int TPW, bool STATE_ONLY>
__global__ __launch_bounds__(256) void recur_scan_kernel(RmiRecurShape s, RmiRecurArgs a, uint32_t n_chunks, uint32_t seg_chunks) {
    __shared__ f32x4 part[2][4][64];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), fr = lane & 15, g = lane >> 4;
    const uint32_t head = blockIdx.y, v0 = blockIdx.x * 16, seg = blockIdx.z, n_tiles = s.d_pad / 16;
    const uint32_t c_begin = seg * seg_chunks, c_end = c_begin + seg_chunks < n_chunks ? c_begin + seg_chunks : n_chunks;
    const RecurScratch ws = recur_scratch_at(a.scratch, s, n_chunks);
    f32x4 st[TPW], kept[TPW];
    const size_t at = size_t(head) * s.d_pad * s.v_pad + v0 + fr, head_state = size_t(s.d_pad) * s.v_pad;
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const uint32_t tile = wave + 4 * i;
        st[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        kept[i] = f32x4{1.f, 1.f, 1.f, 1.f};
        if (STATE_ONLY || tile >= n_tiles) continue;
        if (a.pos0)
#pragma unroll
            for (int r = 0; r < 4; r++) st[i][r] = a.state_in[at + size_t(tile * 16 + g * 4 + r) * s.v_pad];
        for (uint32_t before = 0; before < seg; before++) {
            const float *u = ws.seg_state + size_t(before) * s.heads * head_state + at;
            const f32x4 keep = *reinterpret_cast<const f32x4 *>(ws.seg_decay + (size_t(before) * s.heads + head) * s.d_pad + tile * 16 + g * 4);
#pragma unroll
            for (int r = 0; r < 4; r++) st[i][r] = __builtin_fmaf(st[i][r], keep[r], u[size_t(tile * 16 + g * 4 + r) * s.v_pad]);
        }
    }
    struct Operands {
        f32x4 q[STATE_ONLY ? 1 : TPW], k[TPW], p[TPW];
        f32x4 v;  // v of tokens 4g .. 4g + 3 at this lane's channel
        f32x4 am;
    };
    auto load = [&](uint32_t chunk) {
        Operands x;
        const size_t hc = size_t(head) * n_chunks + chunk;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            const uint32_t tile = wave + 4 * i < n_tiles ? wave + 4 * i : n_tiles - 1;
            if (!STATE_ONLY) x.q[STATE_ONLY ? 0 : i] = *reinterpret_cast<const f32x4 *>(ws.qp + (hc * kChunk + fr) * s.d_pad + tile * 16 + g * 4);
            x.k[i] = *reinterpret_cast<const f32x4 *>(ws.kt + (hc * s.d_pad + tile * 16 + fr) * kChunk + g * 4);
            x.p[i] = *reinterpret_cast<const f32x4 *>(ws.pc + hc * s.d_pad + tile * 16 + g * 4);
        }
        if (!STATE_ONLY) x.am = *reinterpret_cast<const f32x4 *>(ws.am + hc * 256 + fr * 16 + g * 4);
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const uint32_t t = chunk * kChunk + g * 4 + r;
            const bool live = t < a.n_tokens && v0 + fr < s.vdim;
            const float v = a.v[live ? size_t(t) * s.heads * s.vdim + size_t(head) * s.vdim + v0 + fr : 0];
            x.v[r] = live ? v : 0.0f;
        }
        return x;
    };
    constexpr uint32_t kAhead = TPW <= 2 ? 4 : 2;  // chunks whose operands are on their way
    Operands ring[kAhead];
#pragma unroll
    for (uint32_t j = 0; j < kAhead; j++) ring[j] = load(c_begin + j < c_end ? c_begin + j : c_end - 1);
    for (uint32_t chunk0 = c_begin; chunk0 < c_end; chunk0 += kAhead) {
#pragma unroll
        for (uint32_t j = 0; j < kAhead; j++) {
            const uint32_t chunk = chunk0 + j;
            if (chunk >= c_end) break;
            const Operands &x = ring[j];
            f32x4 o[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};  // two chains
            if (!STATE_ONLY && wave == 3) o[0] = mma16_f32(x.am, x.v, o[0]);
#pragma unroll
            for (int i = 0; i < TPW; i++) {
                if (wave + 4 * i >= n_tiles) continue;
                if (!STATE_ONLY) o[(i + 1) & 1] = mma16_f32(x.q[STATE_ONLY ? 0 : i], st[i], o[(i + 1) & 1]);
                st[i] *= x.p[i];
                if (STATE_ONLY) kept[i] *= x.p[i];
                st[i] = mma16_f32(x.k[i], x.v, st[i]);
            }
            ring[j] = load(chunk + kAhead < c_end ? chunk + kAhead : c_end - 1);
            if (STATE_ONLY) continue;
            part[chunk & 1][wave][lane] = o[0] + o[1];
            __syncthreads();  // (two buffers: the next chunk's writes cannot meet this one's reads)
            if (wave == (chunk & 3)) {
                const f32x4 sum = (part[chunk & 1][0][lane] + part[chunk & 1][1][lane]) + (part[chunk & 1][2][lane] + part[chunk & 1][3][lane]);
                float *dst = ws.o + ((size_t(head) * n_chunks + chunk) * kChunk + g * 4) * s.v_pad + v0 + fr;
#pragma unroll
                for (int r = 0; r < 4; r++) dst[size_t(r) * s.v_pad] = sum[r];
            }
        }
    }
    if (!STATE_ONLY && c_end != n_chunks) return;  // the last segment ends with the pass's state
    float *out = STATE_ONLY ? ws.seg_state + size_t(seg) * s.heads * head_state + at : a.state_out + at;
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const uint32_t tile = wave + 4 * i;
        if (tile >= n_tiles) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) out[size_t(tile * 16 + g * 4 + r) * s.v_pad] = st[i][r];
        if (STATE_ONLY && blockIdx.x == 0 && fr == 0)
            *reinterpret_cast<f32x4 *>(ws.seg_decay + (size_t(seg) * s.heads + head) * s.d_pad + tile * 16 + g * 4) = kept[i];
    }
}

// a wave: one (token, head): o over its root mean square, times the weight
template <typename T>
__global__ __launch_bounds__(256) void recur_norm_kernel(RmiRecurShape s, RmiRecurArgs a, uint32_t n_chunks) {
    const uint32_t lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6), head = blockIdx.y;
    if (t >= a.n_tokens) return;
    const float *o = recur_scratch_at(a.scratch, s, n_chunks).o + (size_t(head) * n_chunks * kChunk + t) * s.v_pad;
    float v[kMaxHeadDim / 64], sq = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++) {
        v[j] = lane + j * 64 < s.vdim ? o[lane + j * 64] : 0.0f;
        sq = __builtin_fmaf(v[j], v[j], sq);
    }
    const float r = 1.0f / sqrtf(wave_sum_f32(sq) / float(s.vdim) + s.eps);
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++)
        if (lane + j * 64 < s.vdim)
            static_cast<T *>(a.out)[size_t(t) * a.out_ld + size_t(head) * s.vdim + lane + j * 64] =
                from_f32<T>(v[j] * r * a.norm[lane + j * 64]);
}

// ------------------------------------------------------------------ launches
// Keys over workgroups where the columns alone would not fill the chip; at most kMaxParts parts of 128 keys or more.
constexpr uint32_t kSplitMaxCols = 256;  // per key/value head
void attn_parts(const RmiAttnShape &s, uint32_t n_tokens, uint32_t n_keys, uint32_t *parts, uint32_t *keys_per_part) {
    const uint32_t group = s.heads / s.kv_heads, tiles = (n_tokens * group + 15) / 16;
    // the most that a tile of sixteen columns sees, from a block's edge on
    const uint64_t seen = s.window ? uint64_t(s.window) + 15 / group + 1 + kKeyBlock : n_keys;
    if (seen < n_keys) n_keys = uint32_t(seen);
    const uint32_t slots = s.kv_heads * tiles, cus = uint32_t(rmi_device_cus());
    uint32_t p = (n_keys + 127) / 128;
    const uint32_t fill = (cus + slots - 1) / slots;
    if (p > fill) p = fill;
    if (p > kMaxParts) p = kMaxParts;
    if (slots > kAttnCounters || p < 1) p = 1;
    const uint32_t align = 4 * kKeyBlock;  // each wave whole value blocks
    *keys_per_part = ((n_keys + p - 1) / p + align - 1) / align * align;
    *parts = (n_keys + *keys_per_part - 1) / *keys_per_part;
}

int check_attn(const RmiAttnShape &s, const RmiAttnArgs &a) {
    if (s.dim > kMaxHeadDim || s.vdim > kMaxHeadDim || s.taps == 0 || s.taps > kMaxTaps || s.heads % s.kv_heads || s.rot_dims > s.dim ||
        s.rot_dims % 2 || s.capacity % kKeyBlock || s.dk_pad % 32 || s.dv_pad % 16 || s.dk_pad < s.dim || s.dv_pad < s.vdim ||
        s.dk_pad > kMaxHeadDim || s.dv_pad > kMaxHeadDim || s.capacity == 0 ||
        (uint64_t(a.pos0) + a.n_tokens > s.capacity && (s.window == 0 || uint64_t(s.window) - 1 + a.n_tokens > s.capacity)))
        return rmi_fail(RMI_HIP_E_INVALID, "bad attention shape");
    return RMI_HIP_OK;
}
uint32_t bucket_of(const RmiAttnShape &s) {
    const uint32_t d = s.dk_pad > s.dv_pad ? s.dk_pad : s.dv_pad;
    return d <= 64 ? 64 : d <= 128 ? 128 : 256;
}
size_t split_lds(uint32_t elem_bytes, const RmiAttnShape &s, uint32_t n_tokens) {
    const uint32_t cols = n_tokens * (s.heads / s.kv_heads), live = cols < 16 ? cols : 16;
    const size_t q = size_t(16) * s.dk_pad * elem_bytes, merge = size_t(4) * (32 + live * s.dv_pad) * 4;
    return q > merge ? q : merge;
}

template <typename T>
int attn_pass(const RmiAttnShape &s, const RmiAttnArgs &a, hipStream_t st) {
    const uint32_t n_heads = s.heads + 2 * s.kv_heads, group = s.heads / s.kv_heads, n_cols = a.n_tokens * group;
    const dim3 conv_grid(n_heads, (a.pos0 % kConvRun + a.n_tokens + 4 * kConvRun - 1) / (4 * kConvRun));
    if (conv_pairs_fit(s))
        hipLaunchKernelGGL(conv_rotate_pairs_kernel<T>, conv_grid, dim3(256), 0, st, s, a);
    else
        hipLaunchKernelGGL(conv_rotate_kernel<T>, conv_grid, dim3(256), 0, st, s, a);
    const uint32_t bucket = bucket_of(s);
    if (n_cols <= kSplitMaxCols) {
        uint32_t parts, kpp;
        attn_parts(s, a.n_tokens, a.pos0 + a.n_tokens, &parts, &kpp);
        const dim3 grid(s.kv_heads * ((n_cols + 15) / 16) * parts);
        const size_t lds = split_lds(sizeof(T), s, a.n_tokens);
        auto go = [&](auto kernel) {
            const int rc = rmi_allow_lds(kernel, lds);
            if (rc == RMI_HIP_OK) hipLaunchKernelGGL(kernel, grid, dim3(256), lds, st, s, a, parts, kpp);
            return rc;
        };
        const int rc = bucket == 64 ? go(attn_split_kernel<T, 64>) : bucket == 128 ? go(attn_split_kernel<T, 128>) : go(attn_split_kernel<T, 256>);
        if (rc != RMI_HIP_OK) return rc;
    } else {
        auto go = [&](auto kernel, uint32_t qt) {
            const size_t lds = size_t(4) * qt * 16 * (s.dv_pad + 6) * 4;
            const int rc = rmi_allow_lds(kernel, lds);
            if (rc == RMI_HIP_OK)
                hipLaunchKernelGGL(kernel, dim3((n_cols + 16 * qt - 1) / (16 * qt) * s.kv_heads), dim3(256), lds, st, s, a);
            return rc;
        };
        const int rc = bucket == 64    ? go(attn_pass_kernel<T, 64, 2>, 2)
                       : bucket == 128 ? go(attn_pass_kernel<T, 128, 2>, 2)
                                       : go(attn_pass_kernel<T, 256, 1>, 1);
        if (rc != RMI_HIP_OK) return rc;
    }
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int check_recur(const RmiRecurShape &s) {
    if (s.heads == 0 || s.dim == 0 || s.vdim == 0 || s.dim > kMaxHeadDim || s.vdim > kMaxHeadDim || s.d_pad % 16 || s.v_pad % 16 ||
        s.d_pad < s.dim || s.v_pad < s.vdim || s.d_pad > kMaxHeadDim || s.v_pad > kMaxHeadDim)
        return rmi_fail(RMI_HIP_E_INVALID, "bad recurrence shape");
    return RMI_HIP_OK;
}

template <typename T>
int mixers_step(const RmiAttnShape *as, const RmiAttnArgs *aa, const RmiRecurShape *rs, const RmiRecurArgs *ra, hipStream_t st) {
    const RmiAttnShape s = as ? *as : RmiAttnShape{};
    const RmiAttnArgs a = aa ? *aa : RmiAttnArgs{};
    const RmiRecurShape r = rs ? *rs : RmiRecurShape{};
    const RmiRecurArgs b = ra ? *ra : RmiRecurArgs{};
    uint32_t parts = 1, kpp = 0, blocks = 0;
    size_t lds = 0;
    if (as) {
        attn_parts(s, 1, a.pos0 + 1, &parts, &kpp);
        blocks = s.kv_heads * ((s.heads / s.kv_heads + 15) / 16) * parts;
        lds = split_lds(sizeof(T), s, 1);
    }
    if (rs && recur_step_lds(r) > lds) lds = recur_step_lds(r);
    const dim3 grid(blocks + (rs ? r.heads : 0));
    const uint32_t bucket = as ? bucket_of(s) : 64;
    auto go = [&](auto kernel) {
        const int rc = rmi_allow_lds(kernel, lds);
        if (rc == RMI_HIP_OK) hipLaunchKernelGGL(kernel, grid, dim3(kStepThreads), lds, st, s, a, blocks, parts, kpp, r, b);
        return rc;
    };
    const int rc = bucket == 64 ? go(mixers_step_kernel<T, 64>) : bucket == 128 ? go(mixers_step_kernel<T, 128>) : go(mixers_step_kernel<T, 256>);
    if (rc != RMI_HIP_OK) return rc;
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

}  // namespace

size_t rmi_attn_scratch_bytes(const RmiAttnShape &s) {
    const size_t cols = kSplitMaxCols > s.heads / s.kv_heads ? kSplitMaxCols : s.heads / s.kv_heads;
    const size_t slots = size_t(s.kv_heads) * ((cols + 15) / 16);
    return kAttnCounters * 4 + slots * kMaxParts * attn_part_floats(s.dv_pad) * 4;
}

size_t rmi_recur_scratch_floats(const RmiRecurShape &s, uint32_t max_tokens) {
    const size_t hc = size_t(s.heads) * ((max_tokens + kChunk - 1) / kChunk);
    return hc * (2 * size_t(kChunk) * s.d_pad + kChunk * kChunk + s.d_pad + size_t(kChunk) * s.v_pad) +
           size_t(kMaxSegs) * s.heads * s.d_pad * (s.v_pad + 1);
}

int rmi_attn_pass(uint32_t elem_bytes, const RmiAttnShape &s, const RmiAttnArgs &a, hipStream_t st) {
    if (a.n_tokens == 0) return RMI_HIP_OK;
    const int rc = check_attn(s, a);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? attn_pass<rmi_bf16>(s, a, st) : attn_pass<float>(s, a, st);
}

int rmi_recur_pass(uint32_t elem_bytes, const RmiRecurShape &s, const RmiRecurArgs &a, hipStream_t st) {
    if (a.n_tokens == 0) return RMI_HIP_OK;
    const int rc = check_recur(s);
    if (rc != RMI_HIP_OK) return rc;
    const uint32_t n_chunks = (a.n_tokens + kChunk - 1) / kChunk;
    const size_t lds = (2 * size_t(kChunk) * (s.d_pad + 4) + 1024) * 4;
    hipLaunchKernelGGL(recur_factors_kernel, dim3(n_chunks, s.heads), dim3(256), lds, st, s, a, n_chunks);
    // segments of eight chunks or more, as many as still find an idle compute unit
    const uint32_t columns = s.heads * (s.v_pad / 16);
    uint32_t segs = (2 * uint32_t(rmi_device_cus()) + columns - 1) / columns;
    if (segs > n_chunks / 8) segs = n_chunks / 8;
    if (segs > kMaxSegs) segs = kMaxSegs;
    if (segs < 1) segs = 1;
    const uint32_t seg_chunks = (n_chunks + segs - 1) / segs;
    segs = (n_chunks + seg_chunks - 1) / seg_chunks;
    auto scan = [&](auto state_only, auto whole) {
        if (segs > 1) hipLaunchKernelGGL(state_only, dim3(s.v_pad / 16, s.heads, segs - 1), dim3(256), 0, st, s, a, n_chunks, seg_chunks);
        hipLaunchKernelGGL(whole, dim3(s.v_pad / 16, s.heads, segs), dim3(256), 0, st, s, a, n_chunks, seg_chunks);
    };
    if (s.d_pad <= 64)
        scan(recur_scan_kernel<1, true>, recur_scan_kernel<1, false>);
    else if (s.d_pad <= 128)
        scan(recur_scan_kernel<2, true>, recur_scan_kernel<2, false>);
    else
        scan(recur_scan_kernel<4, true>, recur_scan_kernel<4, false>);
    const dim3 ngrid((a.n_tokens + 3) / 4, s.heads);
    if (elem_bytes == 2)
        hipLaunchKernelGGL(recur_norm_kernel<rmi_bf16>, ngrid, dim3(256), 0, st, s, a, n_chunks);
    else
        hipLaunchKernelGGL(recur_norm_kernel<float>, ngrid, dim3(256), 0, st, s, a, n_chunks);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_mixers_step(uint32_t elem_bytes, const RmiAttnShape *as, const RmiAttnArgs *aa, const RmiRecurShape *rs, const RmiRecurArgs *ra,
                    hipStream_t st) {
    if (!as && !rs) return RMI_HIP_OK;
    int rc = as ? check_attn(*as, *aa) : RMI_HIP_OK;
    if (rc == RMI_HIP_OK && rs) rc = check_recur(*rs);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? mixers_step<rmi_bf16>(as, aa, rs, ra, st) : mixers_step<float>(as, aa, rs, ra, st);
}
