// Minimal gated recurrence: a linear recurrence per channel whose gates read the current token only, so that the tokens of a portion
// compose (S -> a S + b) and are scanned in parallel.
#include "attention_tiles.hpp"
#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_gated_lanes = 0;        // tuning: threads across the channels of a block of the scan, 8 or 16

namespace {

// bf16 models: the native exponential and reciprocal (a few ulp); f32 models: the library's
template <bool FAST>
__device__ __forceinline__ float logistic(float x) {
    if constexpr (FAST) return __builtin_amdgcn_rcpf(1.0f + exp2_fast(-x * kLog2e));
    else return 1.0f / (1.0f + expf(-x));
}

template <int S>
using Piece = float __attribute__((ext_vector_type(S)));

// S channels of an activation row
template <int S, typename T>
__device__ __forceinline__ Piece<S> load_piece(const T *p) {
    if constexpr (sizeof(T) == 4) {
        return *(const Piece<S> *)p;
    } else if constexpr (S == 4) {
        const v2u t = *(const v2u *)p;
        return Piece<S>{bf16_lo(t[0]), bf16_hi(t[0]), bf16_lo(t[1]), bf16_hi(t[1])};
    } else {
        return Piece<S>(bf16_to_f32(*p));
    }
}
template <int S, typename T>
__device__ __forceinline__ void store_piece(T *p, const Piece<S> &v) {
    if constexpr (sizeof(T) == 4) *(Piece<S> *)p = v;
    else if constexpr (S == 4) *(v2u *)p = v2u{f32x2_to_bf16x2(v[0], v[1]), f32x2_to_bf16x2(v[2], v[3])};
    else *p = f32_to_bf16(v[0]);
}

// One token of the recurrence, S -> a S + b
template <int S, bool FAST>
__device__ __forceinline__ void token_step(const Piece<S> &z, const Piece<S> &u, Piece<S> &a, Piece<S> &b) {
#pragma unroll
    for (int e = 0; e < S; ++e) {
        const float c = u[e] >= 0.0f ? u[e] + 0.5f : logistic<FAST>(u[e]);
        if constexpr (FAST) {                        // z = 1 / (1 + t), 1 - z = t z; t stays finite
            const float t = exp2_fast(fminf(-z[e] * kLog2e, 120.0f)), w = __builtin_amdgcn_rcpf(1.0f + t);
            a[e] = t * w;
            b[e] = w * c;
        } else {
            a[e] = logistic<FAST>(-z[e]);
            b[e] = logistic<FAST>(z[e]) * c;
        }
    }
}
template <int S, bool FAST>
__device__ __forceinline__ Piece<S> gated(const Piece<S> &s, const Piece<S> &g, float scale) {
    Piece<S> o;
#pragma unroll
    for (int e = 0; e < S; ++e) o[e] = s[e] * (g[e] * logistic<FAST>(g[e])) * scale;
    return o;
}

// One token per sequence; thread: S channels of a row.
template <typename T, int S>
__global__ void __launch_bounds__(256) gated_step_kernel(GatedIo io, uint32_t width, RaggedRows rr) {
    constexpr bool FAST = sizeof(T) == 2;
    const uint32_t r = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * S;
    if (c >= width) return;
    float *state = io.state + (uint64_t)rr.state_slot[rr.row_seq[r]] * gated_pitch(width) + c;
    const float *row = io.zu + (uint64_t)r * io.ld_zu + c;
    const Piece<S> z = *(const Piece<S> *)row + *(const Piece<S> *)(io.z_bias + c);
    const Piece<S> u = *(const Piece<S> *)(row + width) + *(const Piece<S> *)(io.u_bias + c);
    const Piece<S> g = load_piece<S>((const T *)io.gate + (uint64_t)r * io.ld_gate + c);
    Piece<S> s = Piece<S>(0.0f), a, b;
    if (rr.pos[r] != 0) s = *(const Piece<S> *)state;
    token_step<S, FAST>(z, u, a, b);
#pragma unroll
    for (int e = 0; e < S; ++e) s[e] = fmaf(a[e], s[e], b[e]);
    *(Piece<S> *)state = s;
    store_piece<S>((T *)io.out + (uint64_t)r * io.ld_out + c, gated<S, FAST>(s, g, io.out_scale));
}

// Portions.  A block takes LANES S channels of a sequence and walks its rows in tiles: thread (i, c) has four tokens of S
// channels, composes them, and the tile's thread rows are scanned inside their wavefronts and through LDS.
constexpr int kScanWaves = 8, kScanTokens = 4;
template <typename T, int S, int LANES>
__global__ void __launch_bounds__(kScanWaves * 64) gated_scan_kernel(GatedIo io, uint32_t width, RaggedRows rr) {
    constexpr bool FAST = sizeof(T) == 2;
    constexpr int ROWS = 64 / LANES, kScanTile = kScanWaves * ROWS * kScanTokens;
    typedef Piece<S> P;
    __shared__ P tot_a[2][kScanWaves][LANES], tot_b[2][kScanWaves][LANES];
    const uint32_t q = blockIdx.y, row0 = rr.row_start[q], n = rr.row_start[q + 1] - row0;
    if (n == 0) return;
    const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, lc = lane % LANES, group = lane / LANES;
    const uint32_t c = (blockIdx.x * LANES + lc) * S;
    const bool in = c < width;
    const uint32_t cc = in ? c : 0;
    float *state = io.state + (uint64_t)rr.state_slot[q] * gated_pitch(width) + cc;
    const float *zu = io.zu + (uint64_t)row0 * io.ld_zu + cc;
    const T *gate = (const T *)io.gate + (uint64_t)row0 * io.ld_gate + cc;
    T *out = (T *)io.out + (uint64_t)row0 * io.ld_out + cc;
    const P zb = *(const P *)(io.z_bias + cc), ub = *(const P *)(io.u_bias + cc);
    P carry = P(0.0f);
    if (rr.pos[row0] != 0) carry = *(const P *)state;
    const uint32_t t_own = (wave * ROWS + group) * kScanTokens;
    P z[kScanTokens], u[kScanTokens], g[kScanTokens];
    auto fetch = [&](uint32_t t0) {
#pragma unroll
        for (int i = 0; i < kScanTokens; ++i) {
            const uint32_t t = t0 + t_own + i < n ? t0 + t_own + i : n - 1;       // rows past the portion repeat its last one
            const float *row = zu + (uint64_t)t * io.ld_zu;
            z[i] = *(const P *)row;
            u[i] = *(const P *)(row + width);
            g[i] = load_piece<S>(gate + (uint64_t)t * io.ld_gate);
        }
    };
    fetch(0);
    int buf = 0;
    for (uint32_t t0 = 0; t0 < n; t0 += kScanTile, buf ^= 1) {
        P a[kScanTokens], b[kScanTokens], gs[kScanTokens], A = P(1.0f), B = P(0.0f);
#pragma unroll
        for (int i = 0; i < kScanTokens; ++i) {
            token_step<S, FAST>(z[i] + zb, u[i] + ub, a[i], b[i]);
            gs[i] = g[i];
            if (t0 + t_own + i >= n) {
                a[i] = P(1.0f);
                b[i] = P(0.0f);
            }
#pragma unroll
            for (int e = 0; e < S; ++e) B[e] = fmaf(a[i][e], B[e], b[i][e]);
            A *= a[i];
        }
        if (t0 + kScanTile < n) fetch(t0 + kScanTile);
        // inclusive over the wavefront's thread rows
#pragma unroll
        for (int off = 1; off < ROWS; off *= 2)
#pragma unroll
            for (int e = 0; e < S; ++e) {
                const float pa = __shfl_up(A[e], off * LANES, 64), pb = __shfl_up(B[e], off * LANES, 64);
                if (group >= off) {
                    B[e] = fmaf(A[e], pb, B[e]);
                    A[e] *= pa;
                }
            }
        if (group == ROWS - 1) {
            tot_a[buf][wave][lc] = A;
            tot_b[buf][wave][lc] = B;
        }
        P ea, eb;                                    // of the thread rows before this one
#pragma unroll
        for (int e = 0; e < S; ++e) {
            ea[e] = __shfl_up(A[e], LANES, 64);
            eb[e] = __shfl_up(B[e], LANES, 64);
            if (group == 0) {
                ea[e] = 1.0f;
                eb[e] = 0.0f;
            }
        }
        __syncthreads();
        P s = carry;
#pragma unroll
        for (int w = 0; w < kScanWaves; ++w) {
            if (w == wave) s = carry;
            const P wa = tot_a[buf][w][lc], wb = tot_b[buf][w][lc];
#pragma unroll
            for (int e = 0; e < S; ++e) carry[e] = fmaf(wa[e], carry[e], wb[e]);
        }
#pragma unroll
        for (int e = 0; e < S; ++e) s[e] = fmaf(ea[e], s[e], eb[e]);
#pragma unroll
        for (int i = 0; i < kScanTokens; ++i) {
#pragma unroll
            for (int e = 0; e < S; ++e) s[e] = fmaf(a[i][e], s[e], b[i][e]);
            if (in && t0 + t_own + i < n) store_piece<S>(out + (uint64_t)(t0 + t_own + i) * io.ld_out, gated<S, FAST>(s, gs[i], io.out_scale));
        }
    }
    if (in && tid < LANES) *(P *)state = carry;
}

template <typename T, int S, int LANES>
void launch_scan(uint32_t width, const GatedIo &io, const RaggedRows &rr, hipStream_t s) {
    gated_scan_kernel<T, S, LANES><<<dim3((width + LANES * S - 1) / (LANES * S), rr.batch), kScanWaves * 64, 0, s>>>(io, width, rr);
}
template <typename T, int S>
void launch_gated(uint32_t width, const GatedIo &io, const RaggedRows &rr, uint32_t max_new, int num_cus, hipStream_t s) {
    // 16 lanes read longer pieces of a row; with too few blocks for the device, 8: half the steps in twice the blocks (us for 4 x 2048
    // tokens, width 4096 / 2048, 16, 8, 4 lanes: 108, 127, 180 / 84, 58, 86)
    const bool wide = g_gated_lanes ? g_gated_lanes == 16 : (uint64_t)((width + 16 * S - 1) / (16 * S)) * rr.batch >= (uint64_t)num_cus;
    if (max_new <= 1) gated_step_kernel<T, S><<<dim3((width + 256 * S - 1) / (256 * S), rr.rows), 256, 0, s>>>(io, width, rr);
    else if (wide) launch_scan<T, S, 16>(width, io, rr, s);
    else launch_scan<T, S, 8>(width, io, rr, s);
}

}  // namespace

void gated_mixer(uint32_t width, const GatedIo &io, int is_f32, const RaggedRows &rr, uint32_t max_new, int num_cus, hipStream_t s) {
    if (rr.rows == 0) return;
    const bool vec = width % 4 == 0 && io.ld_zu % 4 == 0 && io.ld_gate % 4 == 0 && io.ld_out % 4 == 0;
    if (is_f32) {
        if (vec) launch_gated<float, 4>(width, io, rr, max_new, num_cus, s);
        else launch_gated<float, 1>(width, io, rr, max_new, num_cus, s);
    } else {
        if (vec) launch_gated<uint16_t, 4>(width, io, rr, max_new, num_cus, s);
        else launch_gated<uint16_t, 1>(width, io, rr, max_new, num_cus, s);
    }
}

}  // namespace k
}  // namespace fa
