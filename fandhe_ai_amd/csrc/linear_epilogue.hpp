// The epilogues of the unquantized linears (LinearEpilogue), shared by their kernels.
#pragma once

#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }

// The value the epilogue makes of y (and, for gate | up, of the up column's y).
template <int MODE>
__device__ __forceinline__ float epilogue_value(const LinearEpilogue &ep, uint32_t row, uint32_t batch, float y, float up) {
    if constexpr (MODE == LinearEpilogue::kGlu) {
        const float g = fminf(y, ep.limit), u = fminf(fmaxf(up, -ep.limit), ep.limit);
        return g * sigmoid_f32(ep.alpha * g) * (u + 1.0f);
    } else if constexpr (MODE == LinearEpilogue::kSiluGlu) {
        return y * sigmoid_f32(y) * up;
    } else if constexpr (MODE == LinearEpilogue::kSoftcap) {
        y *= ep.factor;
        return ep.cap > 0.0f ? ep.cap * tanhf(y / ep.cap) : y;
    } else if constexpr (MODE == LinearEpilogue::kHeadGate) {
        return y * ep.factor * sigmoid_f32(ep.gate[(uint64_t)row * ep.ld_gate + batch]);
    } else if constexpr (MODE == LinearEpilogue::kSquaredRelu) {
        const float r = fmaxf(y, 0.0f);
        return r * r;
    } else if constexpr (MODE == LinearEpilogue::kXielu) {
        return (y > 0.0f ? ep.act[0] * y * y : ep.act[1] * (expm1f(y) - y)) + 0.5f * y;
    } else if constexpr (MODE == LinearEpilogue::kStore) {
        return y * ep.factor;
    } else {
        return y;
    }
}

// Modes whose column tiles alternate gate and up
constexpr bool is_glu(int mode) { return mode == LinearEpilogue::kGlu || mode == LinearEpilogue::kSiluGlu; }

template <int MODE>
__device__ __forceinline__ void epilogue_store1(const LinearEpilogue &ep, uint32_t row, uint32_t col, uint32_t batch, float y, float up) {
    float v = epilogue_value<MODE>(ep, row, batch, y, up);
    if (MODE == LinearEpilogue::kStore && ep.bias) v += ep.bias[col];
    if constexpr (MODE == LinearEpilogue::kResidual) {
        float *o = (float *)ep.out + (uint64_t)row * ep.ld_out + col;
        *o = *o + (ep.scale ? ep.scale[col] * v : v);
        return;
    }
    if (MODE == LinearEpilogue::kStore && col >= ep.n_lo) {
        ep.out_hi[(uint64_t)row * ep.ld_hi + (col - ep.n_lo)] = v;
        return;
    }
    const uint64_t o = batch * ep.out_batch + (uint64_t)row * ep.ld_out + col;
    if (ep.out_f32) ((float *)ep.out)[o] = v;
    else ((uint16_t *)ep.out)[o] = dev::f32_to_bf16(v);
}

// Columns col .. col + 3 of a row (those below n).
template <int MODE>
__device__ __forceinline__ void epilogue_store4(const LinearEpilogue &ep, uint32_t row, uint32_t col, uint32_t n, uint32_t batch,
                                                dev::v4f y, dev::v4f up) {
    const uint64_t o = batch * ep.out_batch + (uint64_t)row * ep.ld_out + col;
    const bool whole = col + 4 <= n && ((ep.ld_out | ep.out_batch) & 3) == 0 && (MODE != LinearEpilogue::kStore || col + 4 <= ep.n_lo);
    if (MODE == LinearEpilogue::kStore && col >= ep.n_lo && col + 4 <= n && ((ep.n_lo | ep.ld_hi) & 3) == 0 && !ep.bias) {
        *(dev::v4f *)(ep.out_hi + (uint64_t)row * ep.ld_hi + (col - ep.n_lo)) = y * ep.factor;
        return;
    }
    if (!whole) {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (col + e < n) epilogue_store1<MODE>(ep, row, col + e, batch, y[e], up[e]);
        return;
    }
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = epilogue_value<MODE>(ep, row, batch, y[e], up[e]);
    if constexpr (MODE == LinearEpilogue::kStore) {
        if (ep.bias) {
            const dev::v4f b = *(const dev::v4f *)(ep.bias + col);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] += b[e];
        }
    }
    if constexpr (MODE == LinearEpilogue::kResidual) {
        dev::v4f *p = (dev::v4f *)((float *)ep.out + o);
        const dev::v4f r = *p, ls = ep.scale ? *(const dev::v4f *)(ep.scale + col) : dev::v4f{1.0f, 1.0f, 1.0f, 1.0f};
        *p = dev::v4f{r[0] + ls[0] * v[0], r[1] + ls[1] * v[1], r[2] + ls[2] * v[2], r[3] + ls[3] * v[3]};
    } else if (ep.out_f32) {
        *(dev::v4f *)((float *)ep.out + o) = dev::v4f{v[0], v[1], v[2], v[3]};
    } else {
        *(dev::v2u *)((uint16_t *)ep.out + o) = dev::v2u{dev::f32x2_to_bf16x2(v[0], v[1]), dev::f32x2_to_bf16x2(v[2], v[3])};
    }
}

// The t-th tile of `tm` rows over all groups (every group's last tile may be part full): its group and index there; false
// behind the last one.  `columns` tiles of columns follow each other inside a group, row tiles fastest.  Every wavefront of
// the block gets the same answer.
__device__ __forceinline__ bool group_tile(const RowGroups &rg, uint32_t t, uint32_t tm, uint32_t columns, uint32_t *group, uint32_t *row_tile,
                                           uint32_t *column) {
    const uint32_t lane = threadIdx.x % 64;
    uint32_t before = 0;
    for (uint32_t g0 = 0; g0 < rg.groups; g0 += 64) {
        const uint32_t own = g0 + lane < rg.groups ? (rg.count[g0 + lane] + tm - 1) / tm : 0;
        uint32_t incl = own;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const uint32_t o = (uint32_t)__shfl_up((int)incl, off, 64);
            if (lane >= (uint32_t)off) incl += o;
        }
        const uint64_t past = __ballot((before + incl) * columns > t);
        if (past) {
            const int first = __builtin_ctzll(past);
            const uint32_t tiles = dev::lane_value(own, first), start = before + dev::lane_value(incl, first) - tiles;
            const uint32_t r = t - start * columns;
            *group = g0 + (uint32_t)first;
            *row_tile = r % tiles;
            *column = r / tiles;
            return true;
        }
        before += dev::lane_value(incl, 63);
    }
    return false;
}

__device__ __forceinline__ uint32_t group_tiles(const RowGroups &rg, uint32_t tm) {
    const uint32_t lane = threadIdx.x % 64;
    uint32_t own = 0;
    for (uint32_t g = lane; g < rg.groups; g += 64) own += (rg.count[g] + tm - 1) / tm;
    return dev::wave_sum(own);
}

}  // namespace k
}  // namespace fa
