// Gated delta rule.  Per head a state S [dim, vdim] in f32, per token
//     S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with q, k unit vectors (q scaled by dim^-1/2), q, k, v behind a short causal convolution and SiLU, and the read-out
// divided by its root mean square, weighted and gated.
#include <algorithm>
#include <type_traits>

#include "device_utils.hpp"
#include "kernels.hpp"
#include "linear_epilogue.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_delta_form = 0;        // tuning: 1 keeps the token-by-token kernel for prompts, 2 takes the chunk form from two tokens on

namespace {

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

__device__ __forceinline__ float log_decay(float a_log, float x) {
    const float sp = x > 0.0f ? x + log1pf(expf(-x)) : log1pf(expf(x));
    return -expf(a_log) * sp;
}

// Convolution + SiLU of channel c for token t of a sequence (row0: its first row of the pass, p: the token's position).
// Inputs before the pass come from the slot's ring.
template <typename T>
__device__ __forceinline__ float conv_silu(const T *__restrict__ y, uint32_t ld, const T *__restrict__ ring, const float *__restrict__ taps,
                                           uint32_t n_taps, uint32_t channels, uint32_t c, uint64_t row0, uint32_t t, uint32_t p) {
    float acc = 0.0f;
    for (uint32_t i = 0; i < n_taps; ++i) {
        const uint32_t back = n_taps - 1 - i;
        if (back > p) continue;                      // before the start
        const float x = back <= t ? load_as_f32(y + (row0 + t - back) * ld + c) : load_as_f32(ring + (uint64_t)((p - back) % n_taps) * channels + c);
        acc = fmaf(taps[(uint64_t)c * n_taps + i], x, acc);
    }
    return silu_f32(acc);
}

// ------------------------------------------------------------------ token by token
// One block per (sequence, head); the state sits in registers (thread: four neighbouring columns of up to RPT rows) from
// the first token of the pass to the last.  CG = column groups of four, a power of two.
template <typename T, int NT, int RPT>
__global__ void __launch_bounds__(NT)
    delta_step_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, uint32_t cg_log2, int write_ring, uint32_t max_tokens) {
    constexpr int NW = NT / 64;
    extern __shared__ float lds[];                   // q [dim], k [dim], v [vdim_p], partial sums [2][RG][CG * 4]
    __shared__ float smem[NW];
    const uint32_t b = blockIdx.x, h = blockIdx.y;
    const uint32_t row0 = rr.row_start[b], n_tok = rr.row_start[b + 1] - row0;
    if (n_tok == 0 || n_tok > max_tokens) return;
    const uint32_t dim = sh.dim, vdim = sh.vdim, vp = sh.vdim_p(), channels = sh.qkv();
    const uint32_t share = sh.heads / sh.kv_heads, hk = h / share;
    const uint32_t CG = 1u << cg_log2, RG = NT >> cg_log2, cg = threadIdx.x & (CG - 1), rg = threadIdx.x >> cg_log2;
    const uint32_t dim_a = (dim + 3) / 4 * 4;        // keeps v and the partial sums 16-byte aligned
    float *lq = lds, *lk = lds + dim_a, *lv = lk + dim_a, *part = lv + CG * 4;
    const T *y = (const T *)io.y;
    T *ring = (T *)io.ring + (uint64_t)rr.state_slot[b] * sh.taps * channels;
    float *state = io.state + ((uint64_t)rr.state_slot[b] * sh.heads + h) * dim * vp;
    const bool col_ok = cg * 4 < vp;
    const uint32_t p0 = (uint32_t)rr.pos[row0];
    v4f S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t d = rg + i * RG;
        S[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (p0 != 0 && col_ok && d < dim) S[i] = *(const v4f *)(state + (uint64_t)d * vp + cg * 4);
    }
    const float a_log = io.a_log[h], dt_bias = io.dt_bias[h];
    for (uint32_t t = 0; t < n_tok; ++t) {
        const uint64_t row = row0 + t;
        const uint32_t p = p0 + t;
        // q, k, v of this head behind the convolution
        float sq = 0.0f, sk = 0.0f;
        for (uint32_t i = threadIdx.x; i < 2 * dim + CG * 4; i += NT) {
            float v = 0.0f;
            if (i < 2 * dim + vdim) {
                const uint32_t c = i < dim ? hk * dim + i : i < 2 * dim ? (sh.kv_heads + hk) * dim + (i - dim) : 2 * sh.kv_heads * dim + h * vdim + (i - 2 * dim);
                v = conv_silu(y, io.ld_y, ring, io.conv, sh.taps, channels, c, row0, t, p);
                if (write_ring && (i >= 2 * dim || h % share == 0)) ring[(uint64_t)(p % sh.taps) * channels + c] = y[row * io.ld_y + c];
            }
            (i < dim ? lq[i] : i < 2 * dim ? lk[i - dim] : lv[i - 2 * dim]) = v;
            if (i < dim) sq = fmaf(v, v, sq);
            else if (i < 2 * dim) sk = fmaf(v, v, sk);
        }
        const float rq = 1.0f / sqrtf(block_sum<float, NW, true>(sq, smem) + 1e-6f) / sqrtf((float)dim);
        const float rk = 1.0f / sqrtf(block_sum<float, NW, true>(sk, smem) + 1e-6f);
        const float beta = sigmoid_f32(io.ba[row * io.ld_ba + h]);
        const float g = expf(log_decay(a_log, io.ba[row * io.ld_ba + sh.heads + h] + dt_bias));
        // S <- g S; S^T k and S^T q of it in one pass
        v4f dk = v4f{0.f, 0.f, 0.f, 0.f}, dq = dk;
        float kq = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const uint32_t d = rg + i * RG;
            if (d >= dim) continue;
            const float kd = lk[d] * rk, qd = lq[d] * rq;
            S[i] *= g;
            dk += S[i] * kd;
            dq += S[i] * qd;
            kq = fmaf(kd, qd, kq);
        }
        ((v4f *)part)[threadIdx.x] = dk;
        ((v4f *)part)[NT + threadIdx.x] = dq;
        // every column group of a row group holds the same share of k . q
        kq = block_sum<float, NW, true>(cg == 0 ? kq : 0.0f, smem);
        dk = dq = v4f{0.f, 0.f, 0.f, 0.f};
        for (uint32_t q = 0; q < RG; ++q) {
            dk += ((const v4f *)part)[(q << cg_log2) + cg];
            dq += ((const v4f *)part)[NT + (q << cg_log2) + cg];
        }
        const v4f u = (*(const v4f *)(lv + cg * 4) - dk) * beta;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const uint32_t d = rg + i * RG;
            if (d < dim) S[i] += u * (lk[d] * rk);
        }
        const v4f o = dq + u * kq;
        float so = 0.0f;
        if (rg == 0) {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (cg * 4 + e < vdim) so = fmaf(o[e], o[e], so);
        }
        const float ro = 1.0f / sqrtf(block_sum<float, NW, true>(so, smem) / (float)vdim + sh.eps);
        if (rg == 0) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const uint32_t c = cg * 4 + e;
                if (c < vdim) {
                    const float gate = load_as_f32(y + row * io.ld_y + channels + h * vdim + c);
                    store_from_f32((T *)io.out + row * io.ld_out + h * vdim + c, o[e] * ro * io.norm[c] * silu_f32(gate));
                }
            }
        }
        __syncthreads();                             // q, k, v and the partial sums are overwritten by the next token
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t d = rg + i * RG;
        if (col_ok && d < dim) *(v4f *)(state + (uint64_t)d * vp + cg * 4) = S[i];
    }
}

// After a pass with more than one token anywhere: the last `taps` inputs of every sequence enter its ring.
template <typename T>
__global__ void __launch_bounds__(256) delta_ring_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr) {
    const uint32_t b = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x, channels = sh.qkv();
    const uint32_t row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0;
    if (c >= channels || n == 0) return;
    T *ring = (T *)io.ring + (uint64_t)rr.state_slot[b] * sh.taps * channels;
    const uint32_t keep = n < sh.taps ? n : sh.taps, p0 = (uint32_t)rr.pos[row0];
    for (uint32_t t = n - keep; t < n; ++t) ring[(uint64_t)((p0 + t) % sh.taps) * channels + c] = ((const T *)io.y)[(uint64_t)(row0 + t) * io.ld_y + c];
}

template <typename T, int NT>
void launch_step(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, uint32_t cg_log2, int write_ring, uint32_t max_tokens, hipStream_t s) {
    const uint32_t rg = NT >> cg_log2, rpt = (sh.dim + rg - 1) / rg;
    const size_t lds = (2 * ((sh.dim + 3) / 4 * 4) + (4u << cg_log2) + 2 * NT * 4) * 4;
    const dim3 grid(rr.batch, sh.heads);
    if (rpt <= 8) delta_step_kernel<T, NT, 8><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens);
    else if (rpt <= 16) delta_step_kernel<T, NT, 16><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens);
    else if (rpt <= 32) delta_step_kernel<T, NT, 32><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens);
    else delta_step_kernel<T, NT, 64><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens);
}

template <typename T>
void mixer(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, uint32_t max_new, hipStream_t s) {
    uint32_t cg_log2 = 0;
    while ((4u << cg_log2) < sh.vdim) ++cg_log2;
    const int write_ring = max_new == 1;
    if (cg_log2 <= 6) launch_step<T, 256>(sh, io, rr, cg_log2, write_ring, max_new, s);
    else launch_step<T, 1024>(sh, io, rr, cg_log2, write_ring, max_new, s);
    if (!write_ring) delta_ring_kernel<T><<<dim3(rr.batch, (sh.qkv() + 255) / 256), 256, 0, s>>>(sh, io, rr);
}

}  // namespace

uint64_t delta_scratch_bytes(const DeltaShape &sh, uint32_t rows, uint32_t batch) { return 0; }

void delta_mixer(const DeltaShape &sh, const DeltaIo &io, int is_f32, const RaggedRows &rr, uint32_t max_new, hipStream_t s) {
    if (rr.rows == 0) return;
    if (is_f32) mixer<float>(sh, io, rr, max_new, s);
    else mixer<uint16_t>(sh, io, rr, max_new, s);
}

}  // namespace k
}  // namespace fa
