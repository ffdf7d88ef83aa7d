// What the launches of the dense products share: checks of their arguments, and the choice of an input's kernel.
#pragma once

#include <type_traits>

#include "device_dense.h"

inline int rmi_check_input(const RmiInput &in, uint32_t k_pad, bool only_x_out) {
    const bool second = in.x2 != nullptr;
    if (!in.x || in.n == 0 || in.n > kInputMax || (in.norm != kNormNone && !in.weight) || (in.y && !in.y_weight) ||
        (only_x_out ? !in.y || !in.x_out : (second ? in.k2 : k_pad) < in.n || k_pad % kDenseKAlign) ||
        (second && (in.norm != kNormNone || in.k2 % kDenseKAlign || in.k2 >= k_pad || k_pad - in.k2 < in.n2)))
        return rmi_fail(RMI_HIP_E_INVALID, "the input does not fit the product");
    return RMI_HIP_OK;
}

inline int rmi_check_row_segs(uint32_t elem_bytes, const RmiDense &w, const RmiRowSegs &segs) {
    bool ok = segs.n_rows == w.n_rows && segs.n_segs > 0 && segs.n_segs <= kMaxRowSegs && w.k_pad % kDenseKAlign == 0 &&
              w.ld == rmi_dense_ld(w.k_pad, elem_bytes);
    for (uint32_t i = 0; ok && i < segs.n_segs; i++)
        ok = (segs.s[i].act == kActReluGlu) == (segs.s[0].act == kActReluGlu) && (segs.s[i].act != kActReluGlu || (segs.s[i].n % 2 == 0 && !segs.s[i].mul)) &&
             (!segs.s[i].mul || (segs.s[i].mul_tok && segs.s[i].mul_rows));
    return ok ? RMI_HIP_OK : rmi_fail(RMI_HIP_E_INVALID, "row segments do not fit the weight");
}

inline int rmi_check_col_segs(uint32_t elem_bytes, const RmiDense &w, const RmiColSegs &segs, uint32_t width) {
    if (w.ld != rmi_dense_ld(w.k_pad, elem_bytes) || segs.n_segs == 0 || segs.n_segs > kMaxColSegs || segs.s[segs.n_segs - 1].k_end != w.k_pad || w.n_rows < width)
        return rmi_fail(RMI_HIP_E_INVALID, "column segments do not fit the weight");
    for (uint32_t i = 0; i < segs.n_segs; i++)
        if (segs.s[i].k_end % kDenseKAlign || segs.s[i].k_end <= (i ? segs.s[i - 1].k_end : 0u))
            return rmi_fail(RMI_HIP_E_INVALID, "column segments do not fit the weight");
    return RMI_HIP_OK;
}

// What a product's row segments ask of its epilogue: each kind is a kernel of its own, so that the plain one stays small.
enum RmiEpilogue : int { kRowsPlain, kRowsActed, kRowsPaired, kRowsTimesTable };
inline RmiEpilogue rmi_epilogue_of(const RmiRowSegs &segs) {
    RmiEpilogue e = kRowsPlain;
    for (uint32_t i = 0; i < segs.n_segs; i++) {
        if (segs.s[i].act == kActReluGlu) return kRowsPaired;
        if (segs.s[i].mul) return kRowsTimesTable;
        if (segs.s[i].act != kActNone) e = kRowsActed;
    }
    return e;
}

// go(norm, add, quads a thread) with the three as compile-time constants
template <typename Go>
int rmi_input_dispatch(const RmiInput &in, Go go) {
    auto quads = [&](auto norm, auto add) {
        if (in.n <= 1024) return go(norm, add, std::integral_constant<int, 1>());
        if (in.n <= 4096) return go(norm, add, std::integral_constant<int, 4>());
        return go(norm, add, std::integral_constant<int, 16>());
    };
    auto added = [&](auto norm) { return in.y ? quads(norm, std::true_type()) : quads(norm, std::false_type()); };
    switch (in.norm) {
        case kNormRms: return added(std::integral_constant<int, kNormRms>());
        case kNormLayer: return added(std::integral_constant<int, kNormLayer>());
        default: return added(std::integral_constant<int, kNormNone>());
    }
}
