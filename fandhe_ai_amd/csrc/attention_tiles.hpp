// Pieces that the attention kernels share: typed element access, and steps of 32 keys on the bf16 matrix instruction with
// scores transposed (keys x query columns), so that the softmax weights are already the next product's operand.
#pragma once

#include <type_traits>

#include "device_utils.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

template <typename T>
__device__ __forceinline__ float load_as_f32(const T *p) {
    if constexpr (std::is_same<T, float>::value) return *p;
    else return bf16_to_f32(*p);
}
template <typename T>
__device__ __forceinline__ void store_from_f32(T *p, float v) {
    if constexpr (std::is_same<T, float>::value) *p = v;
    else *p = f32_to_bf16(v);
}

// The i-th pair of a rotation of 2 half entries: neighbours, or half the entries apart
__device__ __forceinline__ uint2 rotation_pair(uint32_t i, uint32_t half, uint32_t interleaved) {
    return interleaved ? make_uint2(2 * i, 2 * i + 1) : make_uint2(i, i + half);
}

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kKeys = 32;                            // keys per step of the kernels below

typedef short v4s __attribute__((ext_vector_type(4)));
typedef short v8s __attribute__((ext_vector_type(8)));

// The transposed operand of a 32-key step from rows staged in LDS: lane (g, c) gets dim c of 16 dims for keys 4 g .. 4 g + 3
// and 16 + 4 g .. + 3, in the order in which the scores of the two key tiles sit in a lane.  rows: LDS element address of
// (key 0, first dim); pitch in elements.
__device__ __forceinline__ v8bf transposed_keys(const uint16_t *rows, uint32_t pitch, int lane) {
    typedef __attribute__((address_space(3))) v4s *lptr;
    const int g = lane / 16, i = lane % 16;
    const uint16_t *p = rows + (4 * g + i / 4) * pitch + 4 * (i % 4);
    const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lptr)p), hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lptr)(p + 16 * pitch));
    return __builtin_bit_cast(v8bf, v8s{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]});
}

// Loads into these registers complete here: inside a loop that has loads of its own in flight, the compiler would otherwise
// wait for both at the first use of every iteration.
template <int N>
__device__ __forceinline__ void hold(v8bf (&r)[N]) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
        v4u t = __builtin_bit_cast(v4u, r[i]);
        asm volatile("" : "+v"(t));
        r[i] = __builtin_bit_cast(v8bf, t);
    }
}

// 2^x without the detour for subnormal results (weights that small count as zero)
__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }

// Maximum over the four lanes with equal lane % 16, in every one of them.
__device__ __forceinline__ float column_max(float v) {
    const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);      // rows of 16: 0 0 2 2 and 1 1 3 3
    v = fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
    const auto q = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return fmaxf(__uint_as_float(q[0]), __uint_as_float(q[1]));
}

// One online-softmax step of a column (query row): scores of eight keys per lane, lanes with equal lane % 16 share the
// column.  Returns the factor for what was accumulated before; w receives the weights as two bf16 terms whose sum keeps
// about 16 bits of them.
__device__ __forceinline__ float softmax_step(const float (&sc)[8], float &m, float &l, v8bf &w_hi, v8bf &w_lo) {
    float mx = fmaxf(fmaxf(fmaxf(sc[0], sc[1]), fmaxf(sc[2], sc[3])), fmaxf(fmaxf(sc[4], sc[5]), fmaxf(sc[6], sc[7])));
    mx = column_max(mx);
    const float m_new = fmaxf(m, mx), ref = m_new == -INFINITY ? 0.0f : m_new;
    const float fix = exp2_fast(m - ref);
    float sum = 0.0f;
    uint32_t hi[4], lo[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float a = exp2_fast(sc[2 * i] - ref), b = exp2_fast(sc[2 * i + 1] - ref);
        sum += a + b;
        hi[i] = f32x2_to_bf16x2(a, b);
        lo[i] = f32x2_to_bf16x2(a - bf16_lo(hi[i]), b - bf16_hi(hi[i]));
    }
    l = l * fix + sum;
    m = m_new;
    w_hi = __builtin_bit_cast(v8bf, v4u{hi[0], hi[1], hi[2], hi[3]});
    w_lo = __builtin_bit_cast(v8bf, v4u{lo[0], lo[1], lo[2], lo[3]});
    return fix;
}

// The weights of a step that no softmax normalizes: sigmoids of scores in powers of two (-inf: 0), as the same two bf16 terms.
__device__ __forceinline__ void sigmoid_step(const float (&sc)[8], v8bf &w_hi, v8bf &w_lo) {
    uint32_t hi[4], lo[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float a = __builtin_amdgcn_rcpf(1.0f + exp2_fast(-sc[2 * i])), b = __builtin_amdgcn_rcpf(1.0f + exp2_fast(-sc[2 * i + 1]));
        hi[i] = f32x2_to_bf16x2(a, b);
        lo[i] = f32x2_to_bf16x2(a - bf16_lo(hi[i]), b - bf16_hi(hi[i]));
    }
    w_hi = __builtin_bit_cast(v8bf, v4u{hi[0], hi[1], hi[2], hi[3]});
    w_lo = __builtin_bit_cast(v8bf, v4u{lo[0], lo[1], lo[2], lo[3]});
}

}  // namespace k
}  // namespace fa
