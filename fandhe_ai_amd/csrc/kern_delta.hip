// Linear recurrences.  Per head a state S [dim, vdim] in f32; the gated delta rule does per token
//     S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with q, k unit vectors (q scaled by dim^-1/2), q, k, v behind a short causal convolution and SiLU, g one decay per head or one
// per row of S.  Lightning attention is S <- g S + k v^T with constant g and q, k, v behind SiLU only.  The read-out is divided
// by its root mean square (of a head or of all heads), weighted and gated.
#include <algorithm>
#include <type_traits>

#include "attention_tiles.hpp"
#include "device_utils.hpp"
#include "kernels.hpp"
#include "linear_epilogue.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_delta_form = 0;        // tuning: 1 keeps the token-by-token kernel for prompts

namespace {

__device__ __forceinline__ float log_decay(float a_log, float x) {
    const float sp = x > 0.0f ? x + log1pf(expf(-x)) : log1pf(expf(x));
    return -expf(a_log) * sp;
}

// x sigmoid(x) and exp(x) on the hardware's exponential and reciprocal (about one unit in the last place each)
__device__ __forceinline__ float fast_exp(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
__device__ __forceinline__ float fast_silu(float x) { return x * __builtin_amdgcn_rcpf(1.0f + fast_exp(-x)); }
__device__ __forceinline__ float output_gate(uint32_t is_sigmoid, float z) {
    const float s = __builtin_amdgcn_rcpf(1.0f + fast_exp(-z));
    return is_sigmoid ? s : z * s;
}
// log_decay in powers of two.  log(1 + y): a series below 1 / 16 (its first term left out is y^6 / 7 of the value)
__device__ __forceinline__ float fast_log2_decay(float a, float x) {
    const float y = fast_exp(-fabsf(x));
    const float series = y * fmaf(y, fmaf(y, fmaf(y, fmaf(y, fmaf(y, -1.0f / 6, 0.2f), -0.25f), 1.0f / 3), -0.5f), 1.0f);
    const float l1p = y < 0.0625f ? series : __builtin_amdgcn_logf(1.0f + y) * 0.6931471805599453f;
    return a * (fmaxf(x, 0.0f) + l1p);               // a = -exp(A_log) log2(e)
}

// Convolution + SiLU of channel c for token t of a sequence (row0: its first row of the pass, p: the token's position).
// Inputs before the pass come from the slot's ring.
template <typename T>
__device__ __forceinline__ float conv_silu(const T *__restrict__ y, uint32_t ld, const T *__restrict__ ring, const float *__restrict__ taps,
                                           uint32_t n_taps, uint32_t channels, uint32_t c, uint64_t row0, uint32_t t, uint32_t p) {
    if (n_taps == 0) return fast_silu(load_as_f32(y + (row0 + t) * ld + c));
    float acc = 0.0f;
    for (uint32_t i = 0; i < n_taps; ++i) {
        const uint32_t back = n_taps - 1 - i;
        if (back > p) continue;                      // before the start
        const float x = back <= t ? load_as_f32(y + (row0 + t - back) * ld + c) : load_as_f32(ring + (uint64_t)((p - back) % n_taps) * channels + c);
        acc = fmaf(taps[(uint64_t)c * n_taps + i], x, acc);
    }
    return fast_silu(acc);
}

// ------------------------------------------------------------------ token by token
// One block per (sequence, head); the state sits in registers (thread: four neighbouring columns of up to RPT rows) from
// the first token of the pass to the last.  CG = column groups of four, a power of two.
// FAST (single tokens, at most four taps, no more than 2 NT channels): the inputs of the convolution are requested ahead of
// the state, so that the convolution runs while the state travels.
template <typename T, int NT, int RPT, bool FAST, Recurrence KIND>
__global__ void __launch_bounds__(NT)
    delta_step_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, uint32_t cg_log2, int write_ring, uint32_t max_tokens) {
    constexpr int NW = NT / 64;
    extern __shared__ float lds[];                   // q [dim], k [dim], v [vdim_p], partial sums [2][RG][CG * 4], decays [dim]
    constexpr bool CHANNEL = KIND == Recurrence::kChannelDelta, LIGHTNING = KIND == Recurrence::kLightning;
    __shared__ float smem[NW];
    const uint32_t b = blockIdx.x, h = blockIdx.y;
    const uint32_t row0 = rr.row_start[b], n_tok = rr.row_start[b + 1] - row0;
    if (n_tok == 0 || n_tok > max_tokens) return;
    const uint32_t dim = sh.dim, vdim = sh.vdim, vp = sh.vdim_p(), channels = sh.qkv();
    const uint32_t share = sh.heads / sh.kv_heads, hk = h / share;
    const uint32_t CG = 1u << cg_log2, RG = NT >> cg_log2, cg = threadIdx.x & (CG - 1), rg = threadIdx.x >> cg_log2;
    const uint32_t dim_a = (dim + 3) / 4 * 4;        // keeps v and the partial sums 16-byte aligned
    float *lq = lds, *lk = lds + dim_a, *lv = lk + dim_a, *part = lv + CG * 4, *lg = part + 2 * NT * 4;
    const T *y = (const T *)io.y;
    T *ring = (T *)io.ring + (uint64_t)rr.state_slot[b] * sh.taps * channels;
    float *state = io.state + ((uint64_t)rr.state_slot[b] * sh.heads + h) * dim * vp;
    const bool col_ok = cg * 4 < vp;
    const uint32_t p0 = (uint32_t)rr.pos[row0];
    auto channel = [&](uint32_t i) { return i < dim ? hk * dim + i : i < 2 * dim ? (sh.kv_heads + hk) * dim + (i - dim) : 2 * sh.kv_heads * dim + h * vdim + (i - 2 * dim); };
    float xin[2][4], win[2][4];
    if constexpr (FAST) {
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const uint32_t i = threadIdx.x + q * NT;
#pragma unroll
            for (uint32_t back = 0; back < 4; ++back) {
                xin[q][back] = win[q][back] = 0.0f;
                if (i < 2 * dim + vdim && (back < sh.taps || back == 0) && back <= p0) {
                    const uint32_t c = channel(i);
                    xin[q][back] = load_as_f32(back == 0 ? y + (uint64_t)row0 * io.ld_y + c : ring + (uint64_t)((p0 - back) % sh.taps) * channels + c);
                    win[q][back] = sh.taps ? io.conv[(uint64_t)c * sh.taps + sh.taps - 1 - back] : 1.0f;
                }
            }
        }
        __builtin_amdgcn_sched_barrier(0);
    }
    // per-channel decays: thread d owns channel d (dim <= NT)
    static_assert(!CHANNEL || NT >= (int)kDeltaMaxDim, "a thread per channel");
    float decay_in = 0.0f, decay_bias = 0.0f;
    if (CHANNEL && threadIdx.x < dim) {
        decay_in = io.decay[(uint64_t)row0 * io.ld_decay + h * dim + threadIdx.x];
        decay_bias = io.dt_bias[h * dim + threadIdx.x];
    }
    v4f S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const uint32_t d = rg + i * RG;
        S[i] = v4f{0.f, 0.f, 0.f, 0.f};
        if (p0 != 0 && col_ok && d < dim) S[i] = stream_load<true>((const v4f *)(state + (uint64_t)d * vp + cg * 4));
    }
    __builtin_amdgcn_sched_barrier(0);
    const float a_log = LIGHTNING ? 0.0f : io.a_log[h], dt_bias = KIND == Recurrence::kDelta ? io.dt_bias[h] : 0.0f;
    for (uint32_t t = 0; t < n_tok; ++t) {
        const uint64_t row = row0 + t;
        const uint32_t p = p0 + t;
        // q, k, v of this head behind the convolution
        float sq = 0.0f, sk = 0.0f;
#pragma unroll FAST ? 2 : 1
        for (uint32_t q = 0; q < (FAST ? 2u : 0x40000000u); ++q) {
            const uint32_t i = threadIdx.x + q * NT;
            if (i >= 2 * dim + CG * 4) break;
            float v = 0.0f;
            if (i < 2 * dim + vdim) {
                const uint32_t c = channel(i);
                if constexpr (FAST) {
                    float acc = 0.0f;
#pragma unroll
                    for (int back = 3; back >= 0; --back) acc = fmaf(win[q][back], xin[q][back], acc);
                    v = fast_silu(acc);
                } else {
                    v = conv_silu(y, io.ld_y, ring, io.conv, sh.taps, channels, c, row0, t, p);
                }
                if (write_ring && (i >= 2 * dim || h % share == 0)) ring[(uint64_t)(p % sh.taps) * channels + c] = y[row * io.ld_y + c];
            }
            (i < dim ? lq[i] : i < 2 * dim ? lk[i - dim] : lv[i - 2 * dim]) = v;
            if (i < dim) sq = fmaf(v, v, sq);
            else if (i < 2 * dim) sk = fmaf(v, v, sk);
        }
        if constexpr (CHANNEL) {
            if (threadIdx.x < dim) {
                if (t) decay_in = io.decay[row * io.ld_decay + h * dim + threadIdx.x];
                lg[threadIdx.x] = expf(log_decay(a_log, decay_in + decay_bias));
            }
        }
        float rq = 1.0f, rk = 1.0f, beta = 1.0f, g = 1.0f;
        if constexpr (LIGHTNING) {
            g = io.decay[h];
            __syncthreads();
        } else {
            rq = 1.0f / sqrtf(block_sum<float, NW, true>(sq, smem) + 1e-6f) / sqrtf((float)dim);
            rk = 1.0f / sqrtf(block_sum<float, NW, true>(sk, smem) + 1e-6f);
            beta = sigmoid_f32(io.beta[row * io.ld_beta + h]);
            if constexpr (!CHANNEL) g = expf(log_decay(a_log, io.decay[row * io.ld_decay + h] + dt_bias));
        }
        // S <- g S; S^T k and S^T q of it in one pass
        v4f dk = v4f{0.f, 0.f, 0.f, 0.f}, dq = dk;
        float kq = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const uint32_t d = rg + i * RG;
            if (d >= dim) continue;
            const float kd = lk[d] * rk, qd = lq[d] * rq;
            S[i] *= CHANNEL ? lg[d] : g;
            if constexpr (!LIGHTNING) dk += S[i] * kd;
            dq += S[i] * qd;
            kq = fmaf(kd, qd, kq);
        }
        if constexpr (!LIGHTNING) ((v4f *)part)[threadIdx.x] = dk;
        ((v4f *)part)[NT + threadIdx.x] = dq;
        // every column group of a row group holds the same share of k . q
        kq = block_sum<float, NW, true>(cg == 0 ? kq : 0.0f, smem);
        dk = dq = v4f{0.f, 0.f, 0.f, 0.f};
        for (uint32_t q = 0; q < RG; ++q) {
            if constexpr (!LIGHTNING) dk += ((const v4f *)part)[(q << cg_log2) + cg];
            dq += ((const v4f *)part)[NT + (q << cg_log2) + cg];
        }
        const v4f u = LIGHTNING ? *(const v4f *)(lv + cg * 4) : (*(const v4f *)(lv + cg * 4) - dk) * beta;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const uint32_t d = rg + i * RG;
            if (d < dim) S[i] += u * (lk[d] * rk);
            if (t + 1 == n_tok && col_ok && d < dim) __builtin_nontemporal_store(S[i], (v4f *)(state + (uint64_t)d * vp + cg * 4));
        }
        const v4f o = dq + u * kq;
        if (sh.norm_all) {                           // the norm runs over all heads: another launch's
            if (rg == 0) {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (cg * 4 + e < vdim) io.raw[(row * sh.heads + h) * vdim + cg * 4 + e] = o[e];
            }
            __syncthreads();
            continue;
        }
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
                    const float gate = load_as_f32((const T *)io.gate + row * io.ld_gate + h * vdim + c);
                    store_from_f32((T *)io.out + row * io.ld_out + h * vdim + c, o[e] * ro * io.norm[c] * output_gate(sh.gate_sigmoid, gate) * io.out_scale);
                }
            }
        }
        __syncthreads();                             // q, k, v and the partial sums are overwritten by the next token
    }
}

// ------------------------------------------------------------------ chunk form
// Prompts: 32 tokens at a time.  With G_i the running sum of the chunk's log decays, S_0 the state in front of it and
//     A_ij = beta_i exp(G_i - G_j) (k_i . k_j)  for j < i,      T = (I + A)^-1,
// the chunk's writes are U = T diag(beta) V - T diag(beta exp G) K S_0, its read-outs
//     o_i = exp(G_i) S_0^T q_i + sum_{j <= i} exp(G_i - G_j) (q_i . k_j) u_j,
// and the state behind it exp(G_C) S_0 + sum_j exp(G_C - G_j) k_j u_j^T.  delta_chunk_kernel forms everything that does
// not need S_0, for all chunks at once; delta_scan_kernel walks a sequence's chunks with the state in registers.  All
// products run on the f32 matrix instruction v_mfma_f32_16x16x4_f32.
//
// Fragments: 16 x 16 tiles kept as one float4 per lane, 1 KiB.  "A order": lane l holds row l % 16, columns 4 (l / 16) + e
// (the first operand of the instructions e = 0 .. 3, which take the columns 4 g + e of the four lane groups g); "D order":
// lane l holds column l % 16, rows 4 (l / 16) + e, what the instruction leaves, and what serves unchanged as the second
// operand of a product over those rows, columns of the first operand in A order.  Per (chunk, head):
//     [-W: 2 x KT, A][exp(G) Q: 2 x KT, A][(decayed K)^T: KT x 2, A][P: 00, 10, 11, A][T diag(beta) V: 2 x VT, D]
// with W = T diag(beta exp G) K, P the decayed lower triangle of Q K^T, KT and VT the tiles of dim and vdim.  Decays per channel
// stand inside the dot products and add a fragment behind P: the chunk's decay of every channel.  Lightning attention has no W,
// and V itself in the last place.
constexpr int kChunk = 32;
constexpr uint32_t kChunkFrom = 12;          // sequences with fewer new tokens stay with the token-by-token kernel

// Fragments that all value columns of a head use, and where they start
__host__ __device__ constexpr int frag_q(Recurrence kind, int kt) { return kind == Recurrence::kLightning ? 0 : 2 * kt; }
__host__ __device__ constexpr int frag_k(Recurrence kind, int kt) { return frag_q(kind, kt) + 2 * kt; }
__host__ __device__ constexpr int frag_p(Recurrence kind, int kt) { return frag_q(kind, kt) + 4 * kt; }
__host__ __device__ constexpr int shared_frags(Recurrence kind, int kt) { return frag_p(kind, kt) + (kind == Recurrence::kChannelDelta ? 4 : 3); }

struct ChunkPlan {
    uint32_t slots, kt, vt;                  // chunk slots of the pass; tiles of dim (a power of two) and vdim
    uint32_t frags;                          // fragments per (chunk, head)
};
ChunkPlan chunk_plan(const DeltaShape &sh, uint32_t rows, uint32_t batch) {
    ChunkPlan p;
    p.slots = rows / kChunk + batch + 1;
    p.kt = 1;
    while (p.kt * 16 < sh.dim) p.kt *= 2;
    p.vt = (sh.vdim + 15) / 16;
    p.frags = shared_frags(sh.kind, (int)p.kt) + 2 * p.vt;
    return p;
}
// Chunk i of sequence b has slot row_start[b] / 32 + b + i: no two chunks share one.
__device__ __forceinline__ uint32_t slot_base(const RaggedRows &rr, uint32_t b) { return rr.row_start[b] / kChunk + b; }

__device__ __forceinline__ v4f mfma4(const v4f &a, const v4f &b, v4f c) {
#pragma unroll
    for (int e = 0; e < 4; ++e) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], c, 0, 0, 0);
    return c;
}

// silu(convolution) of `cols` channels from c0 on for the chunk's tokens t0 .. into dst [32][pitch]; zeros for tokens past
// the end and columns up to cols_p.  A thread takes TG tokens of two neighbouring channels (one where they are not aligned).
template <typename T, int MAXTAPS, int TG, int NT = 256>
__device__ __forceinline__ void conv_chunk(float *dst, uint32_t pitch, const T *__restrict__ y, uint32_t ld, const T *__restrict__ ring,
                                           const float *__restrict__ conv, uint32_t taps, uint32_t channels, uint32_t c0, uint32_t cols,
                                           uint32_t cols_p, uint64_t row0, uint32_t t0, uint32_t n, uint32_t p0) {
    constexpr uint32_t NG = kChunk / TG;
    if (MAXTAPS != 0 && ((ld | channels | c0 | cols) & 1) == 0) {
        constexpr int NX = TG + (MAXTAPS ? MAXTAPS : 1) - 1, MT = MAXTAPS ? MAXTAPS : 1;
        const uint32_t pairs = cols_p / 2;
        for (uint32_t item = threadIdx.x; item < pairs * NG; item += NT) {
            const uint32_t col = item % pairs * 2, tg = item / pairs * TG;
            const uint32_t c = c0 + (col < cols ? col : 0);
            v2f w[MT], x[NX];
#pragma unroll
            for (int j = 0; j < NX; ++j) {
                const int t = (int)(t0 + tg) + j - (MT - 1);
                const bool inside = t >= 0 && t < (int)n, before = t < 0 && (int)p0 + t >= 0 && -t < (int)taps;
                const T *src = before ? ring + (uint64_t)((p0 + t) % taps) * channels + c : y + (row0 + (inside ? t : 0)) * ld + c;
                v2f v;
                if constexpr (std::is_same<T, float>::value) {
                    v = *(const v2f *)src;
                } else {
                    const uint32_t u = *(const uint32_t *)src;
                    v = v2f{bf16_lo(u), bf16_hi(u)};
                }
                x[j] = inside || before ? v : v2f{0.0f, 0.0f};
            }
#pragma unroll
            for (int i = 0; i < MT; ++i)
#pragma unroll
                for (int e = 0; e < 2; ++e)          // w[back]
                    w[i][e] = i < (int)taps ? conv[(uint64_t)(c + e) * taps + taps - 1 - i] : taps == 0 && i == 0 ? 1.0f : 0.0f;
#pragma unroll
            for (int j = 0; j < TG; ++j) {
                v2f r;
#pragma unroll
                for (int e = 0; e < 2; ++e) {
                    float acc = 0.0f;
#pragma unroll
                    for (int i = MT - 1; i >= 0; --i) acc = fmaf(w[i][e], x[j + MT - 1 - i][e], acc);
                    r[e] = t0 + tg + j < n && col < cols ? fast_silu(acc) : 0.0f;
                }
                *(v2f *)(dst + (tg + j) * pitch + col) = r;
            }
        }
        return;
    }
    for (uint32_t item = threadIdx.x; item < cols_p * NG; item += NT) {
        const uint32_t col = item % cols_p, tg = item / cols_p * TG;
        for (uint32_t j = 0; j < TG; ++j) {
            const uint32_t t = t0 + tg + j;
            dst[(tg + j) * pitch + col] = t < n && col < cols ? conv_silu(y, ld, ring, conv, taps, channels, c0 + col, row0, t, p0 + t) : 0.0f;
        }
    }
}

// lt = T = (I + A)^-1 for the strictly lower A in la (pitch 36), by one wavefront: the diagonal blocks column by column (lanes
// 0 - 15, 16 - 31), then T10 = -T11 A10 T00.
__device__ __forceinline__ void invert_unit_lower(const float *la, float *lt, int lane) {
    const int lr = lane % 16, g = lane / 16;
    if (lane < 32) {
        const int o = (lane / 16) * 16;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float v = i == lr ? 1.0f : 0.0f;
#pragma unroll
            for (int j = 0; j < i; ++j) v = fmaf(-la[(o + i) * 36 + o + j], x[j], v);
            x[i] = v;
            lt[(o + i) * 36 + o + lr] = v;
        }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
    __builtin_amdgcn_wave_barrier();
    v4f x = v4f{0.f, 0.f, 0.f, 0.f}, t00, t10 = x;
#pragma unroll
    for (int e = 0; e < 4; ++e) t00[e] = lt[(4 * g + e) * 36 + lr];
    x = mfma4(*(const v4f *)(la + (16 + lr) * 36 + 4 * g), t00, x);
    t10 = mfma4(*(const v4f *)(lt + (16 + lr) * 36 + 16 + 4 * g), x, t10);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        lt[(16 + 4 * g + e) * 36 + lr] = -t10[e];
        lt[(4 * g + e) * 36 + 16 + lr] = 0.0f;
    }
}

// Fragments of T diag(beta): second operand of W^T, first operand of T V
__device__ __forceinline__ void load_scaled_inverse(v4f (&tf)[2][2], const float *lt, const float *beta, int lr, int g) {
#pragma unroll
    for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
            tf[rt][ct] = *(const v4f *)(lt + (rt * 16 + lr) * 36 + ct * 16 + 4 * g);
#pragma unroll
            for (int e = 0; e < 4; ++e) tf[rt][ct][e] *= beta[ct * 16 + 4 * g + e];
        }
}

// Tile (rt, nt) of T diag(beta) V
__device__ __forceinline__ v4f value_tile(const v4f (&tf)[2][2], const float *lv, uint32_t pitch, uint32_t rt, uint32_t nt, int lr, int g) {
    v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
    for (uint32_t ct = 0; ct <= rt; ++ct) {
        v4f vf;
#pragma unroll
        for (int e = 0; e < 4; ++e) vf[e] = lv[(ct * 16 + 4 * g + e) * pitch + nt * 16 + lr];
        acc = mfma4(rt == 0 ? tf[0][0] : ct == 0 ? tf[1][0] : tf[1][1], vf, acc);
    }
    return acc;
}

// One block per (chunk, q / k head); the heads that share it are taken one after the other.
template <typename T, int KT, int MAXTAPS>
__global__ void __launch_bounds__(256)
    delta_chunk_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, float *__restrict__ frags, float *__restrict__ chunk_decay, uint32_t n_frags) {
    constexpr uint32_t DP = KT * 16, PITCH = DP + 4, VS = 64, VPITCH = VS + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float *lk = lds, *lq = lk + 32 * PITCH, *lv = lq + 32 * PITCH;          // K, Q, 64 columns of V
    float *la = lv + 32 * VPITCH, *lt = la + 32 * 36;                       // A and T, pitch 36
    __shared__ float rq[32], rk[32], beta[32], G[32], qs[32], ks[32], ke[32];   // qs = rq exp(G), ks = rk exp(G), ke = rk exp(G_C - G)
    // the slot's sequence and chunk
    uint32_t lo = 0, hi = rr.batch;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (slot_base(rr, mid) <= blockIdx.x) lo = mid;
        else hi = mid;
    }
    const uint32_t b = lo, row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, t0 = (blockIdx.x - slot_base(rr, b)) * kChunk;
    if (n < kChunkFrom || t0 >= n) return;
    const uint32_t hk = blockIdx.y, share = sh.heads / sh.kv_heads, dim = sh.dim, vdim = sh.vdim, channels = sh.qkv();
    const T *y = (const T *)io.y, *ring = (const T *)io.ring + (uint64_t)rr.state_slot[b] * sh.taps * channels;
    const uint32_t p0 = (uint32_t)rr.pos[row0];
    const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, lr = lane % 16, g = lane / 16;

    conv_chunk<T, MAXTAPS, 8>(lq, PITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, hk * dim, dim, DP, row0, t0, n, p0);
    conv_chunk<T, MAXTAPS, 8>(lk, PITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, (sh.kv_heads + hk) * dim, dim, DP, row0, t0, n, p0);
    __syncthreads();
    {   // four threads per row of Q and of K
        const float *row = (tid < 128 ? lq : lk) + ((tid % 128) / 4) * PITCH;
        float sq = 0.0f;
        for (uint32_t i = tid % 4; i < DP; i += 4) sq = fmaf(row[i], row[i], sq);
        sq += __shfl_xor(sq, 1, 64);
        sq += __shfl_xor(sq, 2, 64);
        if (tid % 4 == 0) {
            const float r = 1.0f / sqrtf(sq + 1e-6f);
            if (tid < 128) rq[tid / 4] = r / sqrtf((float)dim);
            else rk[(tid - 128) / 4] = r;
        }
    }
    // (K K^T) tiles 00, 10, 11 and (K Q^T) tiles: wave 0: both 00, 1: KK 10, 2: QK 10, 3: both 11.  Rows of the result are
    // j (the keys), its column i: D order of the transpose is A order of the matrix.
    auto dot_tile = [&](const float *rows_j, const float *rows_i) {
        v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
        rows_j += lr * PITCH + g;
        rows_i += lr * PITCH + g;
#pragma unroll
        for (uint32_t k = 0; k < DP; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(rows_j[k], rows_i[k], acc, 0, 0, 0);
        return acc;
    };
    const int ti = wave == 0 ? 0 : 1, tj = wave == 3 ? 1 : 0, i_ = ti * 16 + lr;
    v4f kk = v4f{0.f, 0.f, 0.f, 0.f}, qk = kk;
    if (wave != 2) kk = dot_tile(lk + tj * 16 * PITCH, lk + ti * 16 * PITCH);
    if (wave != 1) qk = dot_tile(lk + tj * 16 * PITCH, lq + ti * 16 * PITCH);

    for (uint32_t h = hk * share; h < (hk + 1) * share; ++h) {
        v4f *out = (v4f *)(frags + ((uint64_t)blockIdx.x * sh.heads + h) * n_frags * 256) + lane;
        auto put = [&](uint32_t f, const v4f &v) { out[f * 64] = v; };
        __syncthreads();                             // norms are there; the previous head's scalars and A, T, V are read
        if (tid < 64) {                              // lanes past 31 only keep the scan whole
            const uint32_t t = t0 + lane;
            float lg = 0.0f, be = 0.0f;
            if (lane < 32 && t < n) {
                be = sigmoid_f32(io.beta[(uint64_t)(row0 + t) * io.ld_beta + h]);
                lg = log_decay(io.a_log[h], io.decay[(uint64_t)(row0 + t) * io.ld_decay + h] + io.dt_bias[h]);
            }
#pragma unroll
            for (int off = 1; off < 32; off <<= 1) {
                const float o = __shfl_up(lg, off, 64);
                if (lane >= off) lg += o;
            }
            const float last = __shfl(lg, 31, 64);
            if (lane < 32) {
                beta[lane] = be;
                G[lane] = lg;
                qs[lane] = rq[lane] * expf(lg);
                ks[lane] = rk[lane] * expf(lg);
                ke[lane] = rk[lane] * expf(last - lg);
            }
        }
        __syncthreads();
        if (wave != 2) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = tj * 16 + 4 * g + e;
                la[i_ * 36 + j] = j < i_ ? beta[i_] * fast_exp(G[i_] - G[j]) * rk[i_] * rk[j] * kk[e] : 0.0f;
            }
        }
        if (wave != 1) {
            v4f d;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = tj * 16 + 4 * g + e;
                d[e] = j <= i_ ? fast_exp(G[i_] - G[j]) * rq[i_] * rk[j] * qk[e] : 0.0f;
            }
            put(6 * KT + ti + tj, d);
        }
        // exp(G) Q and the decayed K^T
        for (uint32_t f = wave; f < 2 * KT; f += 4) {
            const uint32_t rt = f / KT, kt = f % KT, i = rt * 16 + lr;
            put(2 * KT + f, *(const v4f *)(lq + i * PITCH + kt * 16 + 4 * g) * qs[i]);
            const uint32_t dt = f / 2, ct = f % 2;
            v4f v;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const uint32_t j = ct * 16 + 4 * g + e;
                v[e] = lk[j * PITCH + dt * 16 + lr] * ke[j];
            }
            put(4 * KT + f, v);
        }
        if (tid == 0) chunk_decay[(uint64_t)blockIdx.x * sh.heads + h] = expf(G[31]);
        // the first columns of V, whose loads travel under the inversion
        const uint32_t vc0 = 2 * sh.kv_heads * dim + h * vdim;
        auto conv_v = [&](uint32_t v0) {
            const uint32_t cols = vdim - v0 < VS ? vdim - v0 : VS;
            conv_chunk<T, MAXTAPS, 4>(lv, VPITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, vc0 + v0, cols, (cols + 15) / 16 * 16, row0, t0, n, p0);
        };
        conv_v(0);
        __syncthreads();
        if (wave == 0) invert_unit_lower(la, lt, lane);
        __syncthreads();
        // -W^T = -K'^T T^T, K' = diag(beta exp(G) rk) K: the columns of the result are tokens, so its D order is W's A order
        v4f tf[2][2];
        load_scaled_inverse(tf, lt, beta, lr, g);
        for (uint32_t f = wave; f < 2 * KT; f += 4) {
            const uint32_t rt = f / KT, kt = f % KT;
            v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
            for (uint32_t ct = 0; ct <= rt; ++ct) {
                v4f kf;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const uint32_t j = ct * 16 + 4 * g + e;
                    kf[e] = -lk[j * PITCH + kt * 16 + lr] * ks[j];
                }
                acc = mfma4(kf, rt == 0 ? tf[0][0] : ct == 0 ? tf[1][0] : tf[1][1], acc);
            }
            put(f, acc);
        }
        // T diag(beta) V
        for (uint32_t v0 = 0; v0 < vdim; v0 += VS) {
            if (v0) {
                __syncthreads();
                conv_v(v0);
                __syncthreads();
            }
            const uint32_t tiles = ((vdim - v0 < VS ? vdim - v0 : VS) + 15) / 16;
            for (uint32_t f = wave; f < 2 * tiles; f += 4) {
                const uint32_t rt = f % 2, nt = f / 2;
                put(6 * KT + 3 + (v0 / 16 + nt) * 2 + rt, value_tile(tf, lv, VPITCH, rt, nt, lr, g));
            }
        }
    }
}

// Decays per channel: G [32][dim].  One block per (chunk, head).  exp(G_i - G_j) is formed from differences that are never
// positive, however strong the decays: pair by pair inside the two diagonal blocks of A and P, and through the last token of the
// first half for the block below the diagonal, exp(G_i - G_15) exp(G_15 - G_j).  G is kept in powers of two.
constexpr int kChannelThreads = 512;
template <typename T, int KT, int MAXTAPS>
__global__ void __launch_bounds__(kChannelThreads) channel_chunk_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, float *__restrict__ frags, uint32_t n_frags) {
    constexpr Recurrence KIND = Recurrence::kChannelDelta;
    constexpr int NT = kChannelThreads, NW = NT / 64;
    constexpr uint32_t DP = KT * 16, PITCH = DP + 4, VS = 64, VPITCH = VS + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float *lk = lds, *lq = lk + 32 * PITCH, *lg = lq + 32 * PITCH, *lv = lg + 32 * PITCH;      // K, Q, G, 64 columns of V
    float *la = lv + 32 * VPITCH, *lt = la + 32 * 36;                       // A, and P then T, pitch 36
    __shared__ float rq[32], rk[32], beta[32];
    uint32_t lo = 0, hi = rr.batch;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (slot_base(rr, mid) <= blockIdx.x) lo = mid;
        else hi = mid;
    }
    const uint32_t b = lo, row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, t0 = (blockIdx.x - slot_base(rr, b)) * kChunk;
    if (n < kChunkFrom || t0 >= n) return;
    const uint32_t h = blockIdx.y, hk = h / (sh.heads / sh.kv_heads), dim = sh.dim, vdim = sh.vdim, channels = sh.qkv();
    const T *y = (const T *)io.y, *ring = (const T *)io.ring + (uint64_t)rr.state_slot[b] * sh.taps * channels;
    const uint32_t p0 = (uint32_t)rr.pos[row0];
    const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, lr = lane % 16, g = lane / 16;
    v4f *out = (v4f *)(frags + ((uint64_t)blockIdx.x * sh.heads + h) * n_frags * 256) + lane;
    auto put = [&](uint32_t f, const v4f &v) { out[f * 64] = v; };

    conv_chunk<T, MAXTAPS, 8, NT>(lq, PITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, hk * dim, dim, DP, row0, t0, n, p0);
    conv_chunk<T, MAXTAPS, 8, NT>(lk, PITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, (sh.kv_heads + hk) * dim, dim, DP, row0, t0, n, p0);
    const float a = -expf(io.a_log[h]) * kLog2e;
    for (uint32_t i = tid; i < 32 * DP; i += NT) {
        const uint32_t t = i / DP, d = i % DP;
        float v = 0.0f;
        if (t0 + t < n && d < dim) v = fast_log2_decay(a, io.decay[(uint64_t)(row0 + t0 + t) * io.ld_decay + h * dim + d] + io.dt_bias[h * dim + d]);
        lg[t * PITCH + d] = v;
    }
    if (tid < 32) beta[tid] = t0 + tid < n ? sigmoid_f32(io.beta[(uint64_t)(row0 + t0 + tid) * io.ld_beta + h]) : 0.0f;
    __syncthreads();
    {   // eight threads per row of Q and of K
        const float *row = (tid < 256 ? lq : lk) + ((tid % 256) / 8) * PITCH;
        float sq = 0.0f;
        for (uint32_t i = tid % 8; i < DP; i += 8) sq = fmaf(row[i], row[i], sq);
#pragma unroll
        for (int off = 1; off < 8; off <<= 1) sq += __shfl_xor(sq, off, 64);
        if (tid % 8 == 0) {
            const float r = 1.0f / sqrtf(sq + 1e-6f);
            if (tid < 256) rq[tid / 8] = r / sqrtf((float)dim);
            else rk[(tid - 256) / 8] = r;
        }
    }
    __syncthreads();
    for (uint32_t d = tid; d < DP; d += NT) {       // running sums, eight tokens read at a time
        float G = 0.0f;
#pragma unroll
        for (uint32_t t1 = 0; t1 < 32; t1 += 8) {
            float v[8];
#pragma unroll
            for (uint32_t t = 0; t < 8; ++t) v[t] = lg[(t1 + t) * PITCH + d];
#pragma unroll
            for (uint32_t t = 0; t < 8; ++t) lg[(t1 + t) * PITCH + d] = G += v[t];
        }
    }
    for (uint32_t i = tid; i < 32 * DP / 4; i += NT) {
        const uint32_t t = i / (DP / 4), d = i % (DP / 4) * 4;
        *(v4f *)(lq + t * PITCH + d) *= rq[t];
        *(v4f *)(lk + t * PITCH + d) *= rk[t];
    }
    __syncthreads();
    // diagonal blocks: wavefronts 0 - 3 a quarter of the channels each of block 0, 4 - 7 of block 1; a lane takes two rows by two
    // columns
    const int blk = wave / 4, part = wave % 4, ti = lane / 8, tj = lane % 8, i0 = blk * 16 + 2 * ti, j0 = blk * 16 + 2 * tj;
    v4f kk = v4f{0.f, 0.f, 0.f, 0.f}, qk = kk;       // (i0, j0), (i0, j0 + 1), (i0 + 1, j0), (i0 + 1, j0 + 1)
    if (tj <= ti) {
        const bool diagonal = ti == tj;
#pragma unroll DP >= 32 ? 2 : 1
        for (uint32_t dd = 0; dd < DP / 4; dd += 4) {
            const uint32_t d = part * (DP / 4) + dd;
            const v4f gi0 = *(const v4f *)(lg + i0 * PITCH + d), gi1 = *(const v4f *)(lg + (i0 + 1) * PITCH + d);
            const v4f gj0 = *(const v4f *)(lg + j0 * PITCH + d), gj1 = *(const v4f *)(lg + (j0 + 1) * PITCH + d);
            const v4f kj0 = *(const v4f *)(lk + j0 * PITCH + d), kj1 = *(const v4f *)(lk + (j0 + 1) * PITCH + d);
            const v4f ki0 = *(const v4f *)(lk + i0 * PITCH + d), ki1 = *(const v4f *)(lk + (i0 + 1) * PITCH + d);
            const v4f qi0 = *(const v4f *)(lq + i0 * PITCH + d), qi1 = *(const v4f *)(lq + (i0 + 1) * PITCH + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float e01 = exp2_fast(fminf(gi0[e] - gj1[e], 0.0f)), e11 = exp2_fast(gi1[e] - gj1[e]), ej = exp2_fast(gj1[e] - gj0[e]);
                const float e00 = diagonal ? 1.0f : e01 * ej, e10 = e11 * ej;
                const float k00 = kj0[e] * e00, k01 = kj1[e] * e01, k10 = kj0[e] * e10, k11 = kj1[e] * e11;
                kk[0] = fmaf(ki0[e], k00, kk[0]);
                kk[1] = fmaf(ki0[e], k01, kk[1]);
                kk[2] = fmaf(ki1[e], k10, kk[2]);
                kk[3] = fmaf(ki1[e], k11, kk[3]);
                qk[0] = fmaf(qi0[e], k00, qk[0]);
                qk[1] = fmaf(qi0[e], k01, qk[1]);
                qk[2] = fmaf(qi1[e], k10, qk[2]);
                qk[3] = fmaf(qi1[e], k11, qk[3]);
            }
        }
    }
    if (part != 0) {                                 // parts 1: in A and P themselves, 2 and 3: in the columns of V
        float *pa = part == 1 ? la : lv + (part - 2) * 1024, *pp = part == 1 ? lt : pa + 512;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int i = 2 * ti + c / 2, j = 2 * tj + c % 2, at = part == 1 ? (blk * 16 + i) * 36 + blk * 16 + j : blk * 256 + i * 16 + j;
            pa[at] = kk[c];
            pp[at] = qk[c];
        }
    }
    if (part == 3) {
        // the block below the diagonal: wavefront 3 of A, 7 of P; the result's rows are keys, its column is a row of the block
        const float *lx = wave == 3 ? lk : lq;
        v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (uint32_t k0 = 0; k0 < DP; k0 += 4) {
            const uint32_t k = k0 + g;
            const float ref = lg[15 * PITCH + k];
            const float kj = lk[lr * PITCH + k] * exp2_fast(ref - lg[lr * PITCH + k]);
            const float xi = lx[(16 + lr) * PITCH + k] * exp2_fast(lg[(16 + lr) * PITCH + k] - ref);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kj, xi, acc, 0, 0, 0);
        }
        float *dst = (wave == 3 ? la : lt) + (16 + lr) * 36 + 4 * g;
        *(v4f *)dst = wave == 3 ? acc * beta[16 + lr] : acc;
    }
    __syncthreads();
    if (part == 0) {
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int i = i0 + c / 2, j = j0 + c % 2, at = blk * 256 + (2 * ti + c / 2) * 16 + 2 * tj + c % 2;
            la[i * 36 + j] = j < i ? beta[i] * ((kk[c] + la[i * 36 + j]) + (lv[at] + lv[1024 + at])) : 0.0f;
            lt[i * 36 + j] = j <= i ? (qk[c] + lt[i * 36 + j]) + (lv[512 + at] + lv[1536 + at]) : 0.0f;
        }
    }
    // exp(G) Q, the decayed K^T, the chunk's decays
    for (uint32_t f = wave; f < 2 * KT; f += NW) {
        const uint32_t rt = f / KT, kt = f % KT, i = rt * 16 + lr;
        const v4f q = *(const v4f *)(lq + i * PITCH + kt * 16 + 4 * g), G = *(const v4f *)(lg + i * PITCH + kt * 16 + 4 * g);
        put(frag_q(KIND, KT) + f, v4f{q[0] * exp2_fast(G[0]), q[1] * exp2_fast(G[1]), q[2] * exp2_fast(G[2]), q[3] * exp2_fast(G[3])});
        const uint32_t dt = f / 2, ct = f % 2, d = dt * 16 + lr;
        const float last = lg[31 * PITCH + d];
        v4f v;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const uint32_t j = ct * 16 + 4 * g + e;
            v[e] = lk[j * PITCH + d] * exp2_fast(last - lg[j * PITCH + d]);
        }
        put(frag_k(KIND, KT) + f, v);
    }
    if (tid < 256)
        frags[(((uint64_t)blockIdx.x * sh.heads + h) * n_frags + frag_p(KIND, KT) + 3) * 256 + tid] = tid < (int)DP ? exp2_fast(lg[31 * PITCH + tid]) : 0.0f;
    const uint32_t vc0 = 2 * sh.kv_heads * dim + h * vdim;
    auto conv_v = [&](uint32_t v0) {
        const uint32_t cols = vdim - v0 < VS ? vdim - v0 : VS;
        conv_chunk<T, MAXTAPS, 4, NT>(lv, VPITCH, y, io.ld_y, ring, io.conv, sh.taps, channels, vc0 + v0, cols, (cols + 15) / 16 * 16, row0, t0, n, p0);
    };
    __syncthreads();                                 // the partial sums are read
    conv_v(0);
    if (wave > 0 && wave < 4) {                      // P: 00, 10, 11
        const int ri = wave == 1 ? 0 : 1, ci = wave == 3 ? 1 : 0;
        put(frag_p(KIND, KT) + wave - 1, *(const v4f *)(lt + (ri * 16 + lr) * 36 + ci * 16 + 4 * g));
    }
    __syncthreads();
    if (wave == 0) invert_unit_lower(la, lt, lane);
    __syncthreads();
    // -W^T = -K'^T T^T, K' = diag(beta) (exp(G) K): the columns of the result are tokens, so its D order is W's A order
    v4f tf[2][2];
    load_scaled_inverse(tf, lt, beta, lr, g);
    for (uint32_t f = wave; f < 2 * KT; f += NW) {
        const uint32_t rt = f / KT, kt = f % KT;
        v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
        for (uint32_t ct = 0; ct <= rt; ++ct) {
            v4f kf;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const uint32_t at = (ct * 16 + 4 * g + e) * PITCH + kt * 16 + lr;
                kf[e] = -lk[at] * exp2_fast(lg[at]);
            }
            acc = mfma4(kf, rt == 0 ? tf[0][0] : ct == 0 ? tf[1][0] : tf[1][1], acc);
        }
        put(f, acc);
    }
    for (uint32_t v0 = 0; v0 < vdim; v0 += VS) {
        if (v0) {
            __syncthreads();
            conv_v(v0);
            __syncthreads();
        }
        const uint32_t tiles = ((vdim - v0 < VS ? vdim - v0 : VS) + 15) / 16;
        for (uint32_t f = wave; f < 2 * tiles; f += NW)
            put(shared_frags(KIND, KT) + (v0 / 16 + f / 2) * 2 + f % 2, value_tile(tf, lv, VPITCH, f % 2, f / 2, lr, g));
    }
}

// Lightning attention: decays d^i are powers of the head's constant; nothing to invert, V stands as it is.
template <typename T, int KT>
__global__ void __launch_bounds__(256)
    lightning_chunk_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, float *__restrict__ frags, float *__restrict__ chunk_decay, uint32_t n_frags) {
    constexpr Recurrence KIND = Recurrence::kLightning;
    constexpr uint32_t DP = KT * 16, PITCH = DP + 4, VS = 64, VPITCH = VS + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float *lk = lds, *lq = lk + 32 * PITCH, *lv = lq + 32 * PITCH;          // K, Q, 64 columns of V
    __shared__ float power[33];                      // d^i
    uint32_t lo = 0, hi = rr.batch;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (slot_base(rr, mid) <= blockIdx.x) lo = mid;
        else hi = mid;
    }
    const uint32_t b = lo, row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, t0 = (blockIdx.x - slot_base(rr, b)) * kChunk;
    if (n < kChunkFrom || t0 >= n) return;
    const uint32_t h = blockIdx.y, hk = h / (sh.heads / sh.kv_heads), dim = sh.dim, vdim = sh.vdim, channels = sh.qkv(), m = n - t0 < kChunk ? n - t0 : kChunk;
    const T *y = (const T *)io.y;
    const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, lr = lane % 16, g = lane / 16;
    v4f *out = (v4f *)(frags + ((uint64_t)blockIdx.x * sh.heads + h) * n_frags * 256) + lane;
    auto put = [&](uint32_t f, const v4f &v) { out[f * 64] = v; };
    if (tid < 33) power[tid] = tid == 0 ? 1.0f : powf(io.decay[h], (float)tid);
    conv_chunk<T, 1, 8>(lq, PITCH, y, io.ld_y, (const T *)nullptr, nullptr, 0, channels, hk * dim, dim, DP, row0, t0, n, 0);
    conv_chunk<T, 1, 8>(lk, PITCH, y, io.ld_y, (const T *)nullptr, nullptr, 0, channels, (sh.kv_heads + hk) * dim, dim, DP, row0, t0, n, 0);
    const uint32_t vc0 = 2 * sh.kv_heads * dim + h * vdim;
    auto load_v = [&](uint32_t v0) {
        const uint32_t cols = vdim - v0 < VS ? vdim - v0 : VS;
        conv_chunk<T, 1, 8>(lv, VPITCH, y, io.ld_y, (const T *)nullptr, nullptr, 0, channels, vc0 + v0, cols, (cols + 15) / 16 * 16, row0, t0, n, 0);
    };
    load_v(0);
    __syncthreads();
    // P: wavefronts 0, 1, 2: 00, 10, 11; rows of the result are keys, D order of the transpose is A order of the matrix
    if (wave < 3) {
        const int ti = wave == 0 ? 0 : 1, tj = wave == 2 ? 1 : 0, i = ti * 16 + lr;
        const float *rows_j = lk + (tj * 16 + lr) * PITCH + g, *rows_i = lq + i * PITCH + g;
        v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (uint32_t k = 0; k < DP; k += 4) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(rows_j[k], rows_i[k], acc, 0, 0, 0);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int j = tj * 16 + 4 * g + e;
            acc[e] = j <= i ? acc[e] * power[i - j] : 0.0f;
        }
        put(frag_p(KIND, KT) + wave, acc);
    }
    for (uint32_t f = wave; f < 2 * KT; f += 4) {
        const uint32_t rt = f / KT, kt = f % KT, i = rt * 16 + lr;
        put(frag_q(KIND, KT) + f, *(const v4f *)(lq + i * PITCH + kt * 16 + 4 * g) * power[i + 1]);
        const uint32_t dt = f / 2, ct = f % 2;
        v4f v;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const uint32_t j = ct * 16 + 4 * g + e;
            v[e] = j < m ? lk[j * PITCH + dt * 16 + lr] * power[m - 1 - j] : 0.0f;
        }
        put(frag_k(KIND, KT) + f, v);
    }
    if (tid == 0) chunk_decay[(uint64_t)blockIdx.x * sh.heads + h] = power[m];
    for (uint32_t v0 = 0; v0 < vdim; v0 += VS) {
        if (v0) {
            __syncthreads();
            load_v(v0);
            __syncthreads();
        }
        const uint32_t tiles = ((vdim - v0 < VS ? vdim - v0 : VS) + 15) / 16;
        for (uint32_t f = wave; f < 2 * tiles; f += 4) {
            v4f v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = lv[(f % 2 * 16 + 4 * g + e) * VPITCH + f / 2 * 16 + lr];
            put(shared_frags(KIND, KT) + (v0 / 16 + f / 2) * 2 + f % 2, v);
        }
    }
}

// LDS buffers of delta_scan_kernel: two where two chunks fit
constexpr int scan_buffers(int kt) { return kt <= 8 ? 2 : 1; }

// One wavefront per (sequence, head, 16 value columns); state tile kt in D order: rows 16 kt + 4 g + e, column l % 16.
template <int KT, Recurrence KIND>
__global__ void __launch_bounds__(512)
    delta_scan_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, const float *__restrict__ frags, const float *__restrict__ chunk_decay,
                      float *__restrict__ o, uint32_t vt, uint32_t n_frags) {
    const int lane = threadIdx.x % 64, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / 64), lr = lane % 16, g = lane / 16;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const uint32_t b = blockIdx.z, h = blockIdx.y, nt_ = blockIdx.x * (blockDim.x / 64) + wave;
    const uint32_t row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0;
    if (n < kChunkFrom) return;
    const bool real = nt_ < vt;                      // a wavefront past the last column tile repeats it and stores nothing
    const uint32_t nt = real ? nt_ : vt - 1;
    const uint32_t dim = sh.dim, vp = sh.vdim_p(), col = nt * 16 + lr, slot0 = slot_base(rr, b), vdim = real ? sh.vdim : 0;
    float *state = io.state + ((uint64_t)rr.state_slot[b] * sh.heads + h) * dim * vp;
    const bool fresh = rr.pos[row0] == 0;
    v4f S[KT];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const uint32_t d = kt * 16 + 4 * g + e;
            S[kt][e] = !fresh && d < dim && col < vdim ? state[(uint64_t)d * vp + col] : 0.0f;
        }
    // A chunk's fragments are staged in LDS as they are (one load instruction moves one fragment), those of the next chunk
    // while this one is multiplied: the shared ones once per block, the values' two per wavefront.
    const uint32_t chunks = (n + kChunk - 1) / kChunk, waves = blockDim.x / 64;
    constexpr int SHARED = shared_frags(KIND, KT), FQ = frag_q(KIND, KT), FK = frag_k(KIND, KT), FP = frag_p(KIND, KT), NB = scan_buffers(KT);
    constexpr bool CHANNEL = KIND == Recurrence::kChannelDelta, LIGHTNING = KIND == Recurrence::kLightning;
    typedef __attribute__((address_space(1))) const void *gptr;
    typedef __attribute__((address_space(3))) void *lptr;
    const uint32_t buf_frags = SHARED + 2 * waves;
    auto stage = [&](uint32_t c, uint32_t buf) {
        const v4f *f = (const v4f *)(frags + ((uint64_t)(slot0 + c) * sh.heads + h) * n_frags * 256) + lane;
        float *l = lds + (uint64_t)buf * buf_frags * 256;
        for (uint32_t i = wave; i < (uint32_t)SHARED; i += waves) __builtin_amdgcn_global_load_lds((gptr)(f + i * 64), (lptr)(l + i * 256), 16, 0, 0);
#pragma unroll
        for (uint32_t i = 0; i < 2; ++i)
            __builtin_amdgcn_global_load_lds((gptr)(f + (SHARED + nt * 2 + i) * 64), (lptr)(l + (SHARED + wave * 2 + i) * 256), 16, 0, 0);
    };
    float decay = CHANNEL ? 1.0f : chunk_decay[(uint64_t)slot0 * sh.heads + h];
    stage(0, 0);
    __builtin_amdgcn_s_waitcnt(0x0F70);              // this wavefront's fragments have landed
    __syncthreads();
    for (uint32_t c = 0; c < chunks; ++c) {
        // the next decay is asked for ahead of the fragments: its use would otherwise wait for all of them
        const float next_decay = CHANNEL ? 1.0f : chunk_decay[(uint64_t)(slot0 + (c + 1 < chunks ? c + 1 : c)) * sh.heads + h];
        if (NB == 2 && c + 1 < chunks) stage(c + 1, (c + 1) & 1);
        const v4f *f = (const v4f *)(lds + (uint64_t)(NB == 2 ? c & 1 : 0) * buf_frags * 256) + lane;
        v4f u[2], r[2] = {v4f{0.f, 0.f, 0.f, 0.f}, v4f{0.f, 0.f, 0.f, 0.f}};
        u[0] = f[(SHARED + wave * 2) * 64];
        u[1] = f[(SHARED + wave * 2 + 1) * 64];
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
            v4f w[2], a[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                if constexpr (!LIGHTNING) w[i] = f[(i * KT + kt) * 64];
                a[i] = f[(FQ + i * KT + kt) * 64];
            }
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int rt = 0; rt < 2; ++rt) {
                    if constexpr (!LIGHTNING) u[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[rt][e], S[kt][e], u[rt], 0, 0, 0);
                    r[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[rt][e], S[kt][e], r[rt], 0, 0, 0);
                }
        }
        r[0] = mfma4(f[FP * 64], u[0], r[0]);
        r[1] = mfma4(f[(FP + 1) * 64], u[0], r[1]);
        r[1] = mfma4(f[(FP + 2) * 64], u[1], r[1]);
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {            // row 16 kt + 4 g + e of the state is element e here
            if constexpr (CHANNEL) S[kt] *= ((const v4f *)(lds + (uint64_t)((NB == 2 ? c & 1 : 0) * buf_frags + FP + 3) * 256))[kt * 4 + g];
            else S[kt] *= decay;
        }
        constexpr int GK = KT < 4 ? KT : 4, GROUPS = 2 * KT / GK;    // fragments are read a group ahead of the multiplies
        v4f kd[2][GK];
        auto read_kd = [&](int q, v4f (&d)[GK]) {
#pragma unroll
            for (int i = 0; i < GK; ++i) d[i] = f[(FK + (q / 2 * GK + i) * 2 + q % 2) * 64];
        };
        read_kd(0, kd[0]);
#pragma unroll
        for (int q = 0; q < GROUPS; ++q) {
            if (q + 1 < GROUPS) read_kd(q + 1, kd[(q + 1) & 1]);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int i = 0; i < GK; ++i)
                    S[q / 2 * GK + i] = __builtin_amdgcn_mfma_f32_16x16x4f32(kd[q & 1][i][e], u[q % 2][e], S[q / 2 * GK + i], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
        auto store = [&]() {
#pragma unroll
            for (int rt = 0; rt < 2; ++rt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const uint32_t t = c * kChunk + rt * 16 + 4 * g + e;
                    if (t < n && col < vdim) o[((uint64_t)(row0 + t) * sh.heads + h) * sh.vdim + col] = r[rt][e];
                }
        };
        if (NB == 1) {
            __syncthreads();
            if (c + 1 < chunks) stage(c + 1, 0);
        }
        __builtin_amdgcn_s_waitcnt(0x0F70);          // the next chunk has landed
        decay = next_decay;
        store();                                     // behind that wait: nothing waits for these stores before the next one
        __syncthreads();                             // ... for everybody, and nobody reads this chunk's any more
    }
    if (!real) return;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const uint32_t d = kt * 16 + 4 * g + e;
            if (d < dim && col < vdim) state[(uint64_t)d * vp + col] = S[kt][e];
        }
}

// Four read-outs, or one: weight, gate, scale, rounding.
template <typename T, typename P>
__device__ __forceinline__ void store_gated(const DeltaShape &sh, P v, const T *gate, T *out) {
    if constexpr (sizeof(P) == 16 && sizeof(T) == 2) {
        const v2u u = *(const v2u *)gate;
        v *= P{output_gate(sh.gate_sigmoid, bf16_lo(u[0])), output_gate(sh.gate_sigmoid, bf16_hi(u[0])), output_gate(sh.gate_sigmoid, bf16_lo(u[1])),
               output_gate(sh.gate_sigmoid, bf16_hi(u[1]))};
        *(v2u *)out = v2u{f32x2_to_bf16x2(v[0], v[1]), f32x2_to_bf16x2(v[2], v[3])};
    } else {
#pragma unroll
        for (int e = 0; e < (int)(sizeof(P) / 4); ++e) store_from_f32(out + e, v[e] * output_gate(sh.gate_sigmoid, load_as_f32(gate + e)));
    }
}

// Read-outs of the chunk form: root mean square, weight, gate.  One wavefront per (row, head); two heads with 32 lanes each where
// four values per lane make a head (HALVES).
template <typename T>
__global__ void __launch_bounds__(256) delta_gate_halves_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr) {
    const uint32_t c = threadIdx.x % 32 * 4, r = blockIdx.x, vdim = sh.vdim, b = rr.row_seq[r];
    if (rr.row_start[b + 1] - rr.row_start[b] < kChunkFrom) return;          // done token by token
    const v4f w = c < vdim ? *(const v4f *)(io.norm + c) * io.out_scale : v4f{0.f, 0.f, 0.f, 0.f};
    for (uint32_t h = threadIdx.x / 32; h < sh.heads; h += 8) {
        const uint64_t at = (uint64_t)r * sh.heads * vdim + h * vdim + c;
        const v4f x = c < vdim ? *(const v4f *)(io.raw + at) : v4f{0.f, 0.f, 0.f, 0.f};
        float sq = row16_sum(fmaf(x[0], x[0], fmaf(x[1], x[1], fmaf(x[2], x[2], x[3] * x[3]))));
        sq += __shfl_xor(sq, 16, 64);
        if (c < vdim)
            store_gated(sh, x * (1.0f / sqrtf(sq / (float)vdim + sh.eps)) * w, (const T *)io.gate + (uint64_t)r * io.ld_gate + h * vdim + c,
                        (T *)io.out + (uint64_t)r * io.ld_out + h * vdim + c);
    }
}
template <typename T>
__global__ void __launch_bounds__(256) delta_gate_kernel(DeltaShape sh, DeltaIo io, RaggedRows rr, const float *__restrict__ o) {
    const uint32_t lane = threadIdx.x % 64, r = blockIdx.x, vdim = sh.vdim, b = rr.row_seq[r];
    if (rr.row_start[b + 1] - rr.row_start[b] < kChunkFrom) return;          // done token by token
    for (uint32_t h = threadIdx.x / 64; h < sh.heads; h += 4) {
        const float *x = o + ((uint64_t)r * sh.heads + h) * vdim;
        float sq = 0.0f;
        for (uint32_t c = lane; c < vdim; c += 64) sq = fmaf(x[c], x[c], sq);
        const float ro = 1.0f / sqrtf(wave_sum_dpp(sq) / (float)vdim + sh.eps);
        const T *gate = (const T *)io.gate + (uint64_t)r * io.ld_gate + h * vdim;
        for (uint32_t c = lane; c < vdim; c += 64)
            store_from_f32((T *)io.out + (uint64_t)r * io.ld_out + h * vdim + c,
                           x[c] * ro * io.norm[c] * output_gate(sh.gate_sigmoid, load_as_f32(gate + c)) * io.out_scale);
    }
}

// The same with the norm over all heads, for every row of the pass.  One block per row; VEC: four values at a time.
template <typename T, int NT, bool VEC>
__global__ void __launch_bounds__(NT) delta_gate_all_kernel(DeltaShape sh, DeltaIo io) {
    constexpr uint32_t S = VEC ? 4 : 1;
    typedef float piece __attribute__((ext_vector_type(S)));
    __shared__ float smem[NT / 64];
    const uint32_t n = sh.heads * sh.vdim;
    const uint64_t r = blockIdx.x;
    const float *x = io.raw + r * n;
    const T *gate = (const T *)io.gate + r * io.ld_gate;
    T *out = (T *)io.out + r * io.ld_out;
    float sq = 0.0f;
    for (uint32_t c = threadIdx.x * S; c < n; c += NT * S) {
        const piece v = *(const piece *)(x + c);
#pragma unroll
        for (int e = 0; e < (int)S; ++e) sq = fmaf(v[e], v[e], sq);
    }
    const float ro = io.out_scale / sqrtf(block_sum<float, NT / 64, true, true>(sq, smem) / (float)n + sh.eps);
    for (uint32_t c = threadIdx.x * S; c < n; c += NT * S) {
        store_gated(sh, *(const piece *)(x + c) * ro * *(const piece *)(io.norm + c), gate + c, out + c);
    }
}

template <typename T>
void gate_all(const DeltaShape &sh, const DeltaIo &io, uint32_t rows, hipStream_t s) {
    const uint32_t n = sh.heads * sh.vdim;
    const bool vec = ((n | io.ld_gate | io.ld_out) & 3) == 0;
    if (rows <= 256 && n > 1024) {
        if (vec) delta_gate_all_kernel<T, 1024, true><<<rows, 1024, 0, s>>>(sh, io);
        else delta_gate_all_kernel<T, 1024, false><<<rows, 1024, 0, s>>>(sh, io);
    } else {
        if (vec) delta_gate_all_kernel<T, 256, true><<<rows, 256, 0, s>>>(sh, io);
        else delta_gate_all_kernel<T, 256, false><<<rows, 256, 0, s>>>(sh, io);
    }
}

// One of a kernel's forms with more LDS than the default limit
template <typename F>
void allow_lds(F f, size_t bytes) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void *>(f), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
}

template <typename T, int KT, Recurrence KIND>
void launch_chunks(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, const ChunkPlan &p, hipStream_t s) {
    float *frags = io.scratch, *decay = frags + (uint64_t)p.slots * sh.heads * p.frags * 256;
    constexpr size_t rows = 32 * (KT * 16 + 4), lds = (rows * (KIND == Recurrence::kChannelDelta ? 3 : 2) + 32 * 68 + 2 * 32 * 36) * 4;
    static bool configured = false;
    auto configure = [&](auto... kernels) {
        if (lds > 65536 && !configured) (allow_lds(kernels, lds), ...);
        configured = true;
    };
    if constexpr (KIND == Recurrence::kDelta) {
        configure(&delta_chunk_kernel<T, KT, 4>, &delta_chunk_kernel<T, KT, 0>);
        auto chunk = sh.taps <= 4 ? &delta_chunk_kernel<T, KT, 4> : &delta_chunk_kernel<T, KT, 0>;
        chunk<<<dim3(p.slots, sh.kv_heads), 256, lds, s>>>(sh, io, rr, frags, decay, p.frags);
    } else if constexpr (KIND == Recurrence::kChannelDelta) {
        configure(&channel_chunk_kernel<T, KT, 4>, &channel_chunk_kernel<T, KT, 0>);
        auto chunk = sh.taps <= 4 ? &channel_chunk_kernel<T, KT, 4> : &channel_chunk_kernel<T, KT, 0>;
        chunk<<<dim3(p.slots, sh.heads), kChannelThreads, lds, s>>>(sh, io, rr, frags, p.frags);
    } else {
        configure(&lightning_chunk_kernel<T, KT>);
        lightning_chunk_kernel<T, KT><<<dim3(p.slots, sh.heads), 256, lds, s>>>(sh, io, rr, frags, decay, p.frags);
    }
    // wavefronts of a block share a head's fragments; fewer per block where there are few blocks
    uint32_t waves = 1;
    while (waves < 8 && waves < p.vt && (uint64_t)rr.batch * sh.heads * ((p.vt + waves - 1) / waves) > 256) waves *= 2;
    const size_t scan_lds = scan_buffers(KT) * (shared_frags(KIND, KT) + 2 * (size_t)waves) * 1024;
    if constexpr (KT >= 2) {
        static bool scan_configured = false;
        if (!scan_configured) allow_lds(&delta_scan_kernel<KT, KIND>, 160 * 1024);
        scan_configured = true;
    }
    delta_scan_kernel<KT, KIND><<<dim3((p.vt + waves - 1) / waves, sh.heads, rr.batch), waves * 64, scan_lds, s>>>(sh, io, rr, frags, decay, io.raw, p.vt, p.frags);
    if (sh.norm_all) return;                         // the whole pass's rows at the end
    if (sh.vdim <= 128 && ((sh.vdim | io.ld_gate | io.ld_out) & 3) == 0) delta_gate_halves_kernel<T><<<rr.rows, 256, 0, s>>>(sh, io, rr);
    else delta_gate_kernel<T><<<rr.rows, 256, 0, s>>>(sh, io, rr, io.raw);
}

template <typename T, Recurrence KIND>
void run_chunks(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, hipStream_t s) {
    const ChunkPlan p = chunk_plan(sh, rr.rows, rr.batch);
    switch (p.kt) {
        case 1: return launch_chunks<T, 1, KIND>(sh, io, rr, p, s);
        case 2: return launch_chunks<T, 2, KIND>(sh, io, rr, p, s);
        case 4: return launch_chunks<T, 4, KIND>(sh, io, rr, p, s);
        case 8: return launch_chunks<T, 8, KIND>(sh, io, rr, p, s);
        default: return launch_chunks<T, 16, KIND>(sh, io, rr, p, s);
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

template <typename T, int NT, Recurrence KIND>
void launch_step(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, uint32_t cg_log2, int write_ring, uint32_t max_tokens, hipStream_t s) {
    const uint32_t rg = NT >> cg_log2, rpt = (sh.dim + rg - 1) / rg;
    const size_t lds = (3 * ((sh.dim + 3) / 4 * 4) + (4u << cg_log2) + 2 * NT * 4) * 4;
    const dim3 grid(rr.batch, sh.heads);
    // FAST's channels fit two per thread by the caller's check
#define FA_STEP(R_)                                                                                                   \
    fast ? delta_step_kernel<T, NT, R_, true, KIND><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens)       \
         : delta_step_kernel<T, NT, R_, false, KIND><<<grid, NT, lds, s>>>(sh, io, rr, cg_log2, write_ring, max_tokens)
    const bool fast = max_tokens == 1 && sh.taps <= 4 && 2 * sh.dim + (4u << cg_log2) <= 2 * NT;
    if (rpt <= 8) FA_STEP(8);
    else if (rpt <= 16) FA_STEP(16);
    else if (rpt <= 32) FA_STEP(32);
    else FA_STEP(64);
#undef FA_STEP
}

template <typename T, Recurrence KIND>
void mixer_kind(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, uint32_t max_new, hipStream_t s) {
    uint32_t cg_log2 = 0;
    while ((4u << cg_log2) < sh.vdim) ++cg_log2;
    const int write_ring = max_new == 1 && sh.taps;
    const bool chunks = max_new >= kChunkFrom && g_delta_form != 1;
    const uint32_t longest = chunks ? kChunkFrom - 1 : max_new;      // sequences of a pass go to one of the two forms by length
    if (!chunks || rr.batch > 1) {
        if (cg_log2 <= 6) launch_step<T, 256, KIND>(sh, io, rr, cg_log2, write_ring, longest, s);
        else launch_step<T, 1024, KIND>(sh, io, rr, cg_log2, write_ring, longest, s);
    }
    if (chunks) run_chunks<T, KIND>(sh, io, rr, s);
    if (!write_ring && sh.taps) delta_ring_kernel<T><<<dim3(rr.batch, (sh.qkv() + 255) / 256), 256, 0, s>>>(sh, io, rr);
    if (sh.norm_all) gate_all<T>(sh, io, rr.rows, s);
}

template <typename T>
void mixer(const DeltaShape &sh, const DeltaIo &io, const RaggedRows &rr, uint32_t max_new, hipStream_t s) {
    switch (sh.kind) {
        case Recurrence::kDelta: return mixer_kind<T, Recurrence::kDelta>(sh, io, rr, max_new, s);
        case Recurrence::kChannelDelta: return mixer_kind<T, Recurrence::kChannelDelta>(sh, io, rr, max_new, s);
        default: return mixer_kind<T, Recurrence::kLightning>(sh, io, rr, max_new, s);
    }
}

}  // namespace

uint64_t delta_scratch_bytes(const DeltaShape &sh, uint32_t rows, uint32_t batch) {
    if (rows < kChunkFrom) return 0;
    const ChunkPlan p = chunk_plan(sh, rows, batch);
    return ((uint64_t)p.slots * sh.heads * (p.frags * 256 + 1) + 64) * 4;
}

void delta_mixer(const DeltaShape &sh, const DeltaIo &io, int is_f32, const RaggedRows &rr, uint32_t max_new, hipStream_t s) {
    if (rr.rows == 0) return;
    if (is_f32) mixer<float>(sh, io, rr, max_new, s);
    else mixer<uint16_t>(sh, io, rr, max_new, s);
}

}  // namespace k
}  // namespace fa
