// Grouped-query attention over paged keys and values for ragged passes: consecutive query heads share a key / value head, keys
// and values have sizes of their own; causal, in a window or over everything; softmax weights, or sigmoids of the scores.
// The query rows of a (sequence, key head) are its (token, head in group) pairs in order; they are the columns of
// S^T = K Q^T, in tiles of 16.
#include <algorithm>

#include "attention_tiles.hpp"
#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_attention_form = 0;     // tuning: 1 the plain kernel, 2 the few-rows kernel for every sequence, 3 the many-rows kernel for every one
int g_attention_blocks = 0;   // tuning: blocks per compute unit the key split aims at

namespace {

// ------------------------------------------------------------------ norms, cache rows
// One block per row of y = q | k | v.  VEC: sizes and pitches allow four values at a time.
template <typename T, int NT, bool VEC>
__global__ void __launch_bounds__(NT)
    attention_prepare_kernel(const float *__restrict__ y, uint32_t ld, const float *__restrict__ q_norm, const float *__restrict__ k_norm,
                             T *__restrict__ q, T *__restrict__ k_pool, T *__restrict__ v_pool, AttentionShape sh,
                             const uint32_t *__restrict__ kv_slot) {
    __shared__ float smem[2][NT / 64];
    constexpr uint32_t S = VEC ? 4 : 1;
    const uint32_t r = blockIdx.x, tid = threadIdx.x, nq = sh.heads * sh.dim, nk = sh.kv_heads * sh.dim, nv = sh.kv_heads * sh.vdim;
    const float *row = y + (uint64_t)r * ld;
    auto squares = [&](const float *v, uint32_t n) {
        float acc = 0.0f;
        for (uint32_t i = tid * S; i < n; i += NT * S) {
            if constexpr (VEC) {
                const v4f t = *(const v4f *)(v + i);
                acc = fmaf(t[0], t[0], fmaf(t[1], t[1], fmaf(t[2], t[2], fmaf(t[3], t[3], acc))));
            } else {
                acc = fmaf(v[i], v[i], acc);
            }
        }
        return acc;
    };
    const uint64_t slot = k_pool ? kv_slot[r] : 0;
    float fq = 1.0f, fk = 1.0f;
    if (q_norm) fq = 1.0f / sqrtf(block_sum<float, NT / 64, true, true>(squares(row, nq), smem[0]) / (float)nq + sh.eps);
    if (k_pool && k_norm) fk = 1.0f / sqrtf(block_sum<float, NT / 64, true, true>(squares(row + nq, nk), smem[1]) / (float)nk + sh.eps);
    auto place = [&](const float *src, uint32_t n, uint32_t size, uint32_t pitch, float f, const float *w, T *dst) {
        for (uint32_t i = tid * S; i < n; i += NT * S) {
            const uint32_t at = size == pitch ? i : i / size * pitch + i % size;
            if constexpr (VEC) {
                v4f t = *(const v4f *)(src + i);
                if (w) {
                    const v4f ww = *(const v4f *)(w + i);
#pragma unroll
                    for (int e = 0; e < 4; ++e) t[e] = t[e] * f * ww[e];
                }
                if constexpr (sizeof(T) == 4) *(v4f *)(dst + at) = t;
                else *(v2u *)(dst + at) = v2u{f32x2_to_bf16x2(t[0], t[1]), f32x2_to_bf16x2(t[2], t[3])};
            } else {
                store_from_f32(dst + at, w ? src[i] * f * w[i] : src[i]);
            }
        }
    };
    place(row, nq, sh.dim, sh.dim_p, fq, q_norm, q + (uint64_t)r * sh.heads * sh.dim_p);
    if (!k_pool || slot >= sh.pool_rows) return;
    place(row + nq, nk, sh.dim, sh.dim_p, fk, k_norm, k_pool + slot * sh.kv_heads * sh.dim_p);
    place(row + nq + nk, nv, sh.vdim, sh.v_p, 1.0f, nullptr, v_pool + slot * sh.kv_heads * sh.v_p);
}

// Norms per head and rotation.  One block per row, or several where there are few rows; groups of 2^group_log2 lanes take one head
// at a time.  VEC: sizes, pitches and the rotated part's halves allow four values at a time.
struct PrepareHeads {
    const float *q_norm, *k_norm, *cos_sin;
    int norms, key_values;
};
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
    attention_prepare_heads_kernel(const float *__restrict__ y, uint32_t ld, PrepareHeads ph, T *__restrict__ q, T *__restrict__ k_pool, T *__restrict__ v_pool,
                                   AttentionShape sh, const uint32_t *__restrict__ kv_slot, const int32_t *__restrict__ pos, uint32_t group_log2) {
    constexpr uint32_t S = VEC ? 4 : 1;
    typedef float piece __attribute__((ext_vector_type(S)));
    const uint32_t r = blockIdx.x, H = sh.heads, G = sh.kv_heads, lanes = 1u << group_log2, lane = threadIdx.x & (lanes - 1);
    const float *row = y + (uint64_t)r * ld, *cs = ph.cos_sin + (uint64_t)r * sh.rot;
    const uint64_t slot = kv_slot[r];
    const uint32_t half = sh.rot / 2;
    auto put = [&](T *dst, const piece &v) {
        if constexpr (sizeof(T) == 4) *(piece *)dst = v;
        else if constexpr (VEC) *(v2u *)dst = v2u{f32x2_to_bf16x2(v[0], v[1]), f32x2_to_bf16x2(v[2], v[3])};
        else *dst = f32_to_bf16(v[0]);
    };
    const uint32_t units = H + (slot < sh.pool_rows ? (ph.key_values ? G : 2 * G) : 0);
    const uint32_t groups = 256u >> group_log2;
    for (uint32_t u = blockIdx.y * groups + (threadIdx.x >> group_log2); u < units; u += gridDim.y * groups) {
        if (u >= H + G) {                            // a value head
            const uint32_t g = u - H - G;
            const float *src = row + (H + G) * sh.dim + g * sh.vdim;
            for (uint32_t i = lane * S; i < sh.vdim; i += lanes * S) put(v_pool + (slot * G + g) * sh.v_p + i, *(const piece *)(src + i));
            continue;
        }
        const float *src = row + u * sh.dim, *w = u < H ? ph.q_norm : ph.k_norm;
        T *dst = u < H ? q + ((uint64_t)r * H + u) * sh.dim_p : k_pool + (slot * G + (u - H)) * sh.dim_p;
        float f = 1.0f;
        if (ph.norms) {
            float sq = 0.0f;
            for (uint32_t i = lane * S; i < sh.dim; i += lanes * S) {
                const piece v = *(const piece *)(src + i);
#pragma unroll
                for (int e = 0; e < (int)S; ++e) sq = fmaf(v[e], v[e], sq);
            }
            for (uint32_t off = lanes / 2; off > 0; off >>= 1) sq += __shfl_xor(sq, (int)off, 64);
            f = 1.0f / sqrtf(sq / (float)sh.dim + sh.eps);
        }
        if (u < H && sh.q_temp != 0.0f) f *= 1.0f + sh.q_temp * logf((float)(((uint32_t)pos[r] + 1) / sh.q_temp_every) + 1.0f);
        auto normed = [&](uint32_t i) {
            piece v = *(const piece *)(src + i) * f;
            if (w) v *= *(const piece *)(w + i);
            return v;
        };
        for (uint32_t i = lane * S; i < sh.dim; i += lanes * S) {
            piece v = normed(i);
            if (i < sh.rot) {
                if (sh.interleaved) {
                    if constexpr (VEC) {
                        const float c0 = cs[i / 2], c1 = cs[i / 2 + 1], s0 = cs[half + i / 2], s1 = cs[half + i / 2 + 1];
                        v = piece{v[0] * c0 - v[1] * s0, v[1] * c0 + v[0] * s0, v[2] * c1 - v[3] * s1, v[3] * c1 + v[2] * s1};
                    } else {
                        const float c = cs[i / 2], s = cs[half + i / 2], o = normed(i ^ 1)[0];
                        v[0] = i & 1 ? v[0] * c + o * s : v[0] * c - o * s;
                    }
                } else {
                    const bool second = i >= half;
                    const uint32_t p = second ? i - half : i;
                    const piece o = normed(second ? p : p + half), c = *(const piece *)(cs + p), s = *(const piece *)(cs + half + p);
                    v = second ? v * c + o * s : v * c - o * s;
                }
            }
            put(dst + i, v);
        }
        if (u >= H && ph.key_values)
            for (uint32_t i = lane * S; i < sh.vdim; i += lanes * S) put(v_pool + (slot * G + (u - H)) * sh.v_p + i, *(const piece *)(src + i));
    }
}

// ------------------------------------------------------------------ output
// Four values of an output head, d .. d + 3: gate, scale, rounding.
struct OutputPlace {
    uint16_t *dst;
    const uint16_t *gate;
};
__device__ __forceinline__ float gate_value(float z) { return 1.0f / (1.0f + expf(-z)); }
// What a (row, head) is multiplied by as a whole
__device__ __forceinline__ float output_scale(const AttentionOutput &ao, uint64_t row, uint32_t head) {
    return ao.head_gate ? ao.scale * gate_value(ao.head_gate[row * ao.ld_head_gate + head]) : ao.scale;
}
__device__ __forceinline__ void store_columns(const OutputPlace &at, uint32_t d, uint32_t vdim, v4f o) {
    if ((vdim & 3) == 0) {
        if (d >= vdim) return;
        if (at.gate) {
            const v2u g = *(const v2u *)(at.gate + d);
            o *= v4f{gate_value(bf16_lo(g[0])), gate_value(bf16_hi(g[0])), gate_value(bf16_lo(g[1])), gate_value(bf16_hi(g[1]))};
        }
        *(v2u *)(at.dst + d) = v2u{f32x2_to_bf16x2(o[0], o[1]), f32x2_to_bf16x2(o[2], o[3])};
        return;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (d + e < vdim) at.dst[d + e] = f32_to_bf16(at.gate ? o[e] * gate_value(bf16_to_f32(at.gate[d + e])) : o[e]);
}
// (row, head) of the output
__device__ __forceinline__ OutputPlace output_place(uint16_t *out, uint32_t ld_out, const AttentionOutput &ao, const AttentionShape &sh, uint64_t row, uint32_t head) {
    return OutputPlace{out + row * ld_out + head * sh.vdim, ao.gate ? (const uint16_t *)ao.gate + row * ao.ld_gate + head * sh.vdim : nullptr};
}

// ------------------------------------------------------------------ plain form: any sizes, f32 or bf16
// One block per (row, head).  Keys are taken 256 at a time, one per thread for the scores, with a running maximum and sum (of a
// softmax); the threads then own value dims.
constexpr uint32_t kPlainMaxV = 4096;
template <typename T>
__global__ void __launch_bounds__(256)
    attention_plain_kernel(const T *__restrict__ q, const T *__restrict__ k_pool, const T *__restrict__ v_pool, T *__restrict__ out, uint32_t ld_out,
                           AttentionOutput ao, AttentionShape sh, RaggedRows rr) {
    extern __shared__ float lq[];                    // the query row
    __shared__ float w[256], smem[4];
    __shared__ uint32_t ids[256];
    const uint32_t r = blockIdx.x, h = blockIdx.y, kh = h / sh.share();
    const uint64_t kw = (uint64_t)sh.kv_heads * sh.dim_p, vw = (uint64_t)sh.kv_heads * sh.v_p;
    const T *qr = q + ((uint64_t)r * sh.heads + h) * sh.dim_p, *kp = k_pool + (uint64_t)kh * sh.dim_p, *vp = v_pool + (uint64_t)kh * sh.v_p;
    for (uint32_t i = threadIdx.x; i < sh.dim; i += 256) lq[i] = load_as_f32(qr + i);
    const int32_t p = rr.pos[r];
    const uint32_t *table = rr.tables + (uint64_t)rr.row_seq[r] * rr.max_blocks;
    float m = -INFINITY, l = 0.0f, acc[kPlainMaxV / 256];
#pragma unroll
    for (uint32_t i = 0; i < kPlainMaxV / 256; ++i) acc[i] = 0.0f;
    bool lost = false;                               // a position without a page: NaN, never a silent zero
    const int32_t first = p - (int32_t)sh.window + 1 > 0 ? p - (int32_t)sh.window + 1 : 0;
    const float slope = ao.slope ? ao.slope[h] : 0.0f, bias = ao.bias ? ao.bias[h] : 0.0f;
    for (int32_t j0 = first; j0 <= p; j0 += 256) {
        __syncthreads();
        const int32_t j = j0 + (int32_t)threadIdx.x;
        float s = -INFINITY;
        uint32_t slot = 0;
        if (j <= p) {
            const uint32_t blk = (uint32_t)j / rr.block_size, id = blk < rr.max_blocks ? table[blk] : 0xffffffffu;
            if (id < rr.num_blocks) {
                slot = id * rr.block_size + (uint32_t)j % rr.block_size;
                const T *key = kp + (uint64_t)slot * kw;
                float d = 0.0f;
                for (uint32_t i = 0; i < sh.dim; ++i) d = fmaf(lq[i], load_as_f32(key + i), d);
                s = d * sh.scale - slope * (float)(p - j) + bias;
            } else {
                s = __uint_as_float(0x7fc00000u);
            }
        }
        ids[threadIdx.x] = slot;
        lost = lost || s != s;
        float fix = 1.0f;
        if (ao.sigmoid) {
            w[threadIdx.x] = j <= p ? gate_value(s) : 0.0f;
            __syncthreads();
        } else {
            const float mc = fmaxf(m, block_max<4, true>(s, smem));
            const float e = j <= p ? expf(s - mc) : 0.0f;
            fix = expf(m - mc);
            w[threadIdx.x] = e;
            l = l * fix + block_sum<float, 4, true>(e, smem);    // its barriers publish w and ids
            m = mc;
        }
        const int32_t n = p - j0 + 1 < 256 ? p - j0 + 1 : 256;
#pragma unroll
        for (uint32_t i = 0; i < kPlainMaxV / 256; ++i) {
            const uint32_t d = threadIdx.x + i * 256;
            if (d >= sh.vdim) continue;
            float a = acc[i] * fix;
            for (int32_t t = 0; t < n; ++t) a = fmaf(w[t], load_as_f32(vp + (uint64_t)ids[t] * vw + d), a);
            acc[i] = a;
        }
    }
    if (ao.sigmoid) l = 1.0f;
    if (__syncthreads_or(lost)) l = __uint_as_float(0x7fc00000u);
    float f = 1.0f;                                  // of what was summed
    if (ao.sink) {
        const float sink = ao.sink[h], mc = fmaxf(m, sink);
        f = expf(m - mc);
        l = l * f + expf(sink - mc);
    }
    f = f / l * output_scale(ao, r, h);
    const T *gate = ao.gate ? (const T *)ao.gate + (uint64_t)r * ao.ld_gate + h * sh.vdim : nullptr;
#pragma unroll
    for (uint32_t i = 0; i < kPlainMaxV / 256; ++i) {
        const uint32_t d = threadIdx.x + i * 256;
        if (d < sh.vdim) store_from_f32(out + (uint64_t)r * ld_out + h * sh.vdim + d, gate ? acc[i] * f * gate_value(load_as_f32(gate + d)) : acc[i] * f);
    }
}

// Whether position p sees key j: 0 <= p - j < W
__device__ __forceinline__ bool seen(int32_t p, int32_t j, int32_t W) { return (uint32_t)(p - j) < (uint32_t)W; }

// Factor of what a column summed with maximum m (of scores in powers of two) and sum l of the weights: the sink takes its share
// of the softmax here.  Sigmoid weights: l is 1 or NaN in every part of the sum.
__device__ __forceinline__ float final_factor(const AttentionOutput &ao, uint64_t row, uint32_t head, float m, float l) {
    const float scale = output_scale(ao, row, head);
    if (ao.sigmoid) return l == l ? scale : l;
    if (!ao.sink) return scale / l;
    const float sink = ao.sink[head] * kLog2e, mx = fmaxf(m, sink), f = exp2f(m - mx);
    return scale * f / (l * f + exp2f(sink - mx));
}

// The scores of a column as sigmoid weights need them, in powers of two: factor a - slope distance + bias
struct ColumnBias {
    float slope, bias;
};
__device__ __forceinline__ ColumnBias column_bias(const AttentionOutput &ao, uint32_t head) {
    return ColumnBias{ao.slope ? ao.slope[head] * kLog2e : 0.0f, ao.bias ? ao.bias[head] * kLog2e : 0.0f};
}
__device__ __forceinline__ float biased(float score, const ColumnBias &cb, int32_t distance) { return fmaf(-cb.slope, (float)distance, score + cb.bias); }

// ------------------------------------------------------------------ few query rows
// A block takes NQ column tiles of one (sequence, key head) and a share of the keys; its wavefronts walk that share 32 keys
// at a time, each on its own: keys go from memory to registers in the operand's order, values through a stage of
// the wavefront's own.  The wavefronts meet in LDS, the blocks of a split in memory.
struct StreamParams {
    const uint16_t *q, *k_pool, *v_pool;
    uint16_t *out;
    uint32_t ld_out;
    AttentionOutput ao;
    float *part_o, *part_ml;                         // [sequence tile][key head][split][16 NQ][v_p], .. [2]: maximum, sum
    uint32_t splits, tiles;                          // tiles of 16 NQ columns per sequence
    uint32_t max_cols;                               // sequences with more columns (and more than one token) are another launch's
};

// D, V: dim_p and v_p in units of 32.
template <int D, int V, int NQ, int NW, bool SIGMOID>
__global__ void __launch_bounds__(NW * 64) attention_stream_kernel(StreamParams p, AttentionShape sh, RaggedRows rr) {
    constexpr int VT = 2 * V, VP = V * 32 + 8, OP = V * 32 + 4;
    constexpr int CPR = V * 4, RPI = 64 / CPR, NV = kKeys / RPI;      // 16-byte pieces of a value row, rows per load, loads per step
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    const uint32_t b = blockIdx.x / p.tiles, tile = blockIdx.x % p.tiles, kh = blockIdx.y, S = sh.share(), G = sh.kv_heads;
    const uint32_t row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, n_cols = n * S, c0 = tile * 16 * NQ;
    if (c0 >= n_cols || (n_cols > p.max_cols && n > 1)) return;
    const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), g = lane / 16, c = lane % 16;
    const uint32_t *table = rr.tables + (uint64_t)b * rr.max_blocks;
    const int32_t p0 = rr.pos[row0];
    const uint32_t last_col = c0 + 16 * NQ - 1 < n_cols ? c0 + 16 * NQ - 1 : n_cols - 1;
    const int32_t W = (int32_t)sh.window, p_lo = p0 + (int32_t)(c0 / S);
    int32_t k_lo = p_lo - W + 1 > 0 ? p_lo - W + 1 : 0, k_hi = p0 + (int32_t)(last_col / S) + 1;      // keys seen by some column
    const uint64_t part = (((uint64_t)blockIdx.x * G + kh) * p.splits + blockIdx.z) * 16 * NQ;
    if (p.splits > 1) {
        const int32_t unit = kKeys * NW / 2, per = ((k_hi - k_lo + (int32_t)p.splits - 1) / (int32_t)p.splits + unit - 1) / unit * unit;
        k_lo += (int32_t)blockIdx.z * per;
        k_hi = k_lo + per < k_hi ? k_lo + per : k_hi;
        if (k_lo >= k_hi) {                          // a split without keys (never the only one)
            if (tid < 16 * NQ) {
                p.part_ml[2 * (part + tid)] = -INFINITY;
                p.part_ml[2 * (part + tid) + 1] = 0.0f;
            }
            return;
        }
    }
    const int32_t k_last = k_hi - 1, first = k_lo + wave * kKeys;
    const uint64_t kw = (uint64_t)G * sh.dim_p, vw = (uint64_t)G * sh.v_p;
    const uint16_t *kp = p.k_pool + (uint64_t)kh * (D * 32) + 8 * g, *vp = p.v_pool + (uint64_t)kh * (V * 32) + (lane % CPR) * 8;
    // lane (g, c) looks up keys c and 16 + c of a step; keys past the walk repeat its last one (their weight is zero)
    uint32_t lost = 0;
    auto page_of = [&](int32_t j) -> uint32_t {
        j = j <= k_last ? j : k_last;
        const uint32_t blk = (uint32_t)j / rr.block_size;
        return blk < rr.max_blocks ? table[blk] : 0xffffffffu;
    };
    auto slot_of = [&](int32_t j, uint32_t id) -> uint32_t {
        j = j <= k_last ? j : k_last;
        if (id >= rr.num_blocks) {
            lost = 1;
            return 0;
        }
        return id * rr.block_size + (uint32_t)j % rr.block_size;
    };
    v8bf kf[2][D];
    v4u vr[NV];
    auto fetch = [&](int32_t k0, uint32_t id0, uint32_t id1) {
        const uint32_t s0 = slot_of(k0 + c, id0), s1 = slot_of(k0 + 16 + c, id1);
#pragma unroll
        for (int s = 0; s < D; ++s) {
            kf[0][s] = __builtin_bit_cast(v8bf, stream_load<true>((const v4u *)(kp + s0 * kw + s * 32)));
            kf[1][s] = __builtin_bit_cast(v8bf, stream_load<true>((const v4u *)(kp + s1 * kw + s * 32)));
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int r = i * RPI + lane / CPR;
            const uint32_t t0 = (uint32_t)__shfl((int)s0, r % 16, 64), t1 = (uint32_t)__shfl((int)s1, r % 16, 64);
            vr[i] = stream_load<true>((const v4u *)(vp + (r < 16 ? t0 : t1) * vw));
        }
    };
    v8bf qf[NQ][D];
    int32_t pos[NQ];
    float m[NQ], l[NQ];
    ColumnBias cb[NQ];
    v4f o[NQ][VT];
    const bool any = first < k_hi;
    uint32_t id0 = 0, id1 = 0;
    if (any) {
        id0 = page_of(first + c);
        id1 = page_of(first + 16 + c);
    }
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        const uint32_t col = c0 + qi * 16 + c, qc = col < n_cols ? col : n_cols - 1, t = qc / S;
        pos[qi] = p0 + (int32_t)t;
        const uint16_t *src = p.q + ((uint64_t)(row0 + t) * sh.heads + kh * S + qc % S) * (D * 32) + 8 * g;
#pragma unroll
        for (int s = 0; s < D; ++s) qf[qi][s] = *(const v8bf *)(src + s * 32);
        m[qi] = SIGMOID ? 0.0f : -INFINITY;
        l[qi] = SIGMOID ? 1.0f : 0.0f;
        if constexpr (SIGMOID) cb[qi] = column_bias(p.ao, kh * S + qc % S);
#pragma unroll
        for (int t2 = 0; t2 < VT; ++t2) o[qi][t2] = v4f{0.f, 0.f, 0.f, 0.f};
    }
    const float factor = sh.scale * kLog2e;
    if (any) {
        fetch(first, id0, id1);
        id0 = page_of(first + NW * kKeys + c);
        id1 = page_of(first + NW * kKeys + 16 + c);
#pragma unroll
        for (int qi = 0; qi < NQ; ++qi) hold(qf[qi]);
    }
    uint16_t *stage = lds + wave * kKeys * VP;
    for (int32_t k0 = first; k0 < k_hi; k0 += NW * kKeys) {
#pragma unroll
        for (int i = 0; i < NV; ++i) *(v4u *)(stage + (i * RPI + lane / CPR) * VP + (lane % CPR) * 8) = vr[i];
        float sc[NQ][8];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            v4f acc[NQ];
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) acc[qi] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < D; ++s)
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi) acc[qi] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[kt][s], qf[qi][s], acc[qi], 0, 0, 0);
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int32_t j = k0 + kt * 16 + 4 * g + e;
                    float v = acc[qi][e] * factor;
                    if constexpr (SIGMOID) v = biased(v, cb[qi], pos[qi] - j);
                    sc[qi][kt * 4 + e] = seen(pos[qi], j, W) && j < k_hi ? v : -INFINITY;
                }
        }
        __builtin_amdgcn_sched_barrier(0);
        if (k0 + NW * kKeys < k_hi) {
            fetch(k0 + NW * kKeys, id0, id1);
            id0 = page_of(k0 + 2 * NW * kKeys + c);
            id1 = page_of(k0 + 2 * NW * kKeys + 16 + c);
        }
        __builtin_amdgcn_sched_barrier(0);
        v8bf w_hi[NQ], w_lo[NQ];
#pragma unroll
        for (int qi = 0; qi < NQ; ++qi) {
            if constexpr (SIGMOID) {
                sigmoid_step(sc[qi], w_hi[qi], w_lo[qi]);
            } else {
                const float fix = softmax_step(sc[qi], m[qi], l[qi], w_hi[qi], w_lo[qi]);
                if (__any(fix != 1.0f)) {
#pragma unroll
                    for (int t = 0; t < VT; ++t) o[qi][t] *= fix;
                }
            }
        }
#pragma unroll
        for (int t = 0; t < VT; ++t) {
            const v8bf v = transposed_keys(stage + t * 16, VP, lane);
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) {
                o[qi][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w_hi[qi], o[qi][t], 0, 0, 0);
                o[qi][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w_lo[qi], o[qi][t], 0, 0, 0);
            }
        }
        // the next step's rows overwrite the stage: its reads above have to be complete, and stay above
        __builtin_amdgcn_wave_barrier();
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        if constexpr (!SIGMOID) {
            l[qi] += __shfl_xor(l[qi], 16, 64);
            l[qi] += __shfl_xor(l[qi], 32, 64);
        }
        if (__any(lost != 0)) l[qi] = __uint_as_float(0x7fc00000u);  // a position without a page: NaN, never a silent zero
    }
    // pairs of wavefronts meet, half of them left over every time
    float *xo = (float *)lds, *xm = xo + NW / 2 * 16 * NQ * OP;
#pragma unroll
    for (int half = NW / 2; half >= 1; half /= 2) {
        __syncthreads();
        if (wave >= half && wave < 2 * half) {
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) {
                const int at = (wave - half) * 16 * NQ + qi * 16 + c;
                if (g == 0) {
                    xm[at * 2] = m[qi];
                    xm[at * 2 + 1] = l[qi];
                }
#pragma unroll
                for (int t = 0; t < VT; ++t) *(v4f *)(xo + at * OP + t * 16 + 4 * g) = o[qi][t];
            }
        }
        __syncthreads();
        if (wave < half) {
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) {
                const int at = wave * 16 * NQ + qi * 16 + c;
                const float m1 = xm[at * 2], l1 = xm[at * 2 + 1], mx = fmaxf(m[qi], m1), ref = mx == -INFINITY ? 0.0f : mx;
                const float f0 = SIGMOID ? 1.0f : exp2f(m[qi] - ref), f1 = SIGMOID ? 1.0f : exp2f(m1 - ref);
                m[qi] = mx;
                l[qi] = SIGMOID ? l[qi] * l1 : l[qi] * f0 + l1 * f1;
#pragma unroll
                for (int t = 0; t < VT; ++t) o[qi][t] = o[qi][t] * f0 + *(const v4f *)(xo + at * OP + t * 16 + 4 * g) * f1;
            }
        }
    }
    if (wave != 0) return;
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        const uint32_t col = c0 + qi * 16 + c;
        if (p.splits > 1) {
            const uint64_t at = part + qi * 16 + c;
            if (g == 0) {
                p.part_ml[2 * at] = m[qi];
                p.part_ml[2 * at + 1] = l[qi];
            }
            if (col < n_cols) {
#pragma unroll
                for (int t = 0; t < VT; ++t) *(v4f *)(p.part_o + at * (V * 32) + t * 16 + 4 * g) = o[qi][t];
            }
        } else if (col < n_cols) {
            const uint32_t head = kh * S + col % S;
            const OutputPlace at = output_place(p.out, p.ld_out, p.ao, sh, row0 + col / S, head);
            const float f = final_factor(p.ao, row0 + col / S, head, m[qi], l[qi]);
#pragma unroll
            for (int t = 0; t < VT; ++t) store_columns(at, t * 16 + 4 * g, sh.vdim, o[qi][t] * f);
        }
    }
}

// Adds the splits of a tile's columns: one wavefront per column, four dims per lane.
constexpr uint32_t kMaxSplits = 64;
__global__ void __launch_bounds__(64) attention_merge_kernel(StreamParams p, AttentionShape sh, RaggedRows rr, uint32_t tile_cols) {
    const uint32_t b = blockIdx.x / p.tiles, tile = blockIdx.x % p.tiles, kh = blockIdx.y, S = sh.share(), lane = threadIdx.x;
    const uint32_t row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, n_cols = n * S, col = tile * tile_cols + blockIdx.z;
    if (col >= n_cols || (n_cols > p.max_cols && n > 1)) return;
    const uint64_t at = ((uint64_t)blockIdx.x * sh.kv_heads + kh) * p.splits * tile_cols + blockIdx.z;
    float ms = -INFINITY, ls = 0.0f;                 // sum 0: the split holds none of the column's keys
    if (lane < p.splits) {
        const v2f v = *(const v2f *)(p.part_ml + 2 * (at + (uint64_t)lane * tile_cols));
        ms = v[0];
        ls = v[1];
    }
    const uint32_t head = kh * S + col % S;
    const float m = wave_max_dpp(ms), f = ls != 0.0f ? exp2f(ms - m) : 0.0f, w = f * final_factor(p.ao, row0 + col / S, head, m, wave_sum_dpp(ls * f));
    const OutputPlace out = output_place(p.out, p.ld_out, p.ao, sh, row0 + col / S, head);
    for (uint32_t d = lane * 4; d < sh.v_p; d += 256) {
        const float *src = p.part_o + at * sh.v_p + d;
        v4f a = v4f{0.f, 0.f, 0.f, 0.f};
        for (uint32_t s0 = 0; s0 < p.splits; s0 += 8) {
            v4f t[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) t[i] = *(const v4f *)(src + (uint64_t)(s0 + i < p.splits ? s0 + i : p.splits - 1) * tile_cols * sh.v_p);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float ws = s0 + i < p.splits ? lane_value(w, (int)(s0 + i)) : 0.0f;
                if (ws != 0.0f) a += t[i] * ws;
            }
        }
        store_columns(out, d, sh.vdim, a);
    }
}

// ------------------------------------------------------------------ many query rows
// A block of four wavefronts takes 64 NQ columns of one (sequence, key head), every wavefront 16 NQ of them, and walks the keys
// they see 32 at a time; K and V of a step are staged in LDS, two stages.
template <int D, int V, int NQ, bool SIGMOID>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(3)))
    attention_flash_kernel(const uint16_t *__restrict__ q, const uint16_t *__restrict__ k_pool, const uint16_t *__restrict__ v_pool,
                           uint16_t *__restrict__ out, uint32_t ld_out, AttentionOutput ao, uint32_t max_cols, AttentionShape sh, RaggedRows rr) {
    constexpr int VT = 2 * V, KP = D * 32 + 8, VP = V * 32 + 8, PK = D / 2, PV = V / 2, BC = 64 * NQ;
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    uint16_t *ks = lds, *vs = lds + 2 * kKeys * KP;  // [2][32][KP], [2][32][VP]
    const uint32_t S = sh.share(), G = sh.kv_heads, kh = blockIdx.y;
    // longest walks first: the last tiles of a sequence
    uint32_t lo = 0, hi = rr.batch;
    const uint32_t slot = gridDim.x - 1 - blockIdx.x;
    auto base = [&](uint32_t b) { return (uint32_t)((uint64_t)rr.row_start[b] * S / BC) + b; };
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (base(mid) <= slot) lo = mid;
        else hi = mid;
    }
    const uint32_t b = lo, row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, n_cols = n * S, c0 = (slot - base(b)) * BC;
    if (c0 >= n_cols || n_cols <= max_cols || (n == 1 && max_cols)) return;
    const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), g = lane / 16, c = lane % 16;
    const uint32_t *table = rr.tables + (uint64_t)b * rr.max_blocks;
    const int32_t p0 = rr.pos[row0];
    auto pos_of = [&](uint32_t col) { return p0 + (int32_t)((col < n_cols ? col : n_cols - 1) / S); };
    const int32_t W = (int32_t)sh.window, k_hi = pos_of(c0 + BC - 1) + 1, p_lo = pos_of(c0), k_lo = p_lo - W + 1 > 0 ? p_lo - W + 1 : 0;
    v8bf qf[NQ][D];
    int32_t pos[NQ];
    ColumnBias cb[NQ];
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        const uint32_t col = c0 + (wave * NQ + qi) * 16 + c, qc = col < n_cols ? col : n_cols - 1;
        pos[qi] = pos_of(col);
        if constexpr (SIGMOID) cb[qi] = column_bias(ao, kh * S + qc % S);
        const uint16_t *src = q + ((uint64_t)(row0 + qc / S) * sh.heads + kh * S + qc % S) * (D * 32) + 8 * g;
#pragma unroll
        for (int s = 0; s < D; ++s) qf[qi][s] = *(const v8bf *)(src + s * 32);
    }
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) hold(qf[qi]);
    const int32_t w_lo_pos = pos_of(c0 + wave * 16 * NQ), w_hi_pos = pos_of(c0 + (wave + 1) * 16 * NQ - 1);

    // staging: eight threads per key, 16 bytes each at a time; keys past the walk repeat its last one (masked)
    const int key = tid / 8, part = tid % 8;
    const uint64_t kw = (uint64_t)G * (D * 32), vw = (uint64_t)G * (V * 32);
    v4u sk[PK], sv[PV];
    auto page_of = [&](int32_t j) -> uint32_t {
        j = j < k_hi ? j : k_hi - 1;
        const uint32_t blk = (uint32_t)j / rr.block_size;
        return blk < rr.max_blocks ? table[blk] : 0xffffffffu;
    };
    auto fetch = [&](int32_t j, uint32_t id) {
        j = j < k_hi ? j : k_hi - 1;
        const bool ok = id < rr.num_blocks;
        const uint64_t slot = (uint64_t)(ok ? id : 0) * rr.block_size + (uint32_t)j % rr.block_size;
        const uint16_t *kr = k_pool + slot * kw + kh * (D * 32) + part * 8, *vr = v_pool + slot * vw + kh * (V * 32) + part * 8;
#pragma unroll
        for (int i = 0; i < PK; ++i) sk[i] = *(const v4u *)(kr + i * 64);
#pragma unroll
        for (int i = 0; i < PV; ++i) sv[i] = *(const v4u *)(vr + i * 64);
        if (!ok) sk[0] = v4u{0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u};      // no page: NaN, never a silent zero
    };
    auto put = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PK; ++i) *(v4u *)(ks + (buf * kKeys + key) * KP + (part + 8 * i) * 8) = sk[i];
#pragma unroll
        for (int i = 0; i < PV; ++i) *(v4u *)(vs + (buf * kKeys + key) * VP + (part + 8 * i) * 8) = sv[i];
    };
    const float factor = sh.scale * kLog2e;
    float m[NQ], l[NQ];
    v4f o[NQ][VT];
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        m[qi] = -INFINITY;
        l[qi] = 0.0f;
#pragma unroll
        for (int t = 0; t < VT; ++t) o[qi][t] = v4f{0.f, 0.f, 0.f, 0.f};
    }
    uint32_t id = page_of(k_lo + key);
    fetch(k_lo + key, id);
    id = page_of(k_lo + kKeys + key);
    put(0);
    __syncthreads();
    int buf = 0;
    for (int32_t k0 = k_lo; k0 < k_hi; k0 += kKeys, buf ^= 1) {
        const bool more = k0 + kKeys < k_hi;
        if (more) {
            fetch(k0 + kKeys + key, id);
            id = page_of(k0 + 2 * kKeys + key);
        }
        if (k0 <= w_hi_pos && k0 + kKeys > w_lo_pos - W + 1) {       // some column of this wavefront sees some key of the step
            const bool inside = k0 + kKeys - 1 <= w_lo_pos && k0 > w_hi_pos - W;       // every column sees every key
            const uint16_t *kb = ks + buf * kKeys * KP, *vb = vs + buf * kKeys * VP;
            float sc[NQ][8];
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                v4f acc[NQ];
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi) acc[qi] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < D; ++s) {
                    const v8bf kf = *(const v8bf *)(kb + (kt * 16 + c) * KP + s * 32 + 8 * g);
#pragma unroll
                    for (int qi = 0; qi < NQ; ++qi) acc[qi] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qi][s], acc[qi], 0, 0, 0);
                }
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        float v = acc[qi][e] * factor;
                        if constexpr (SIGMOID) v = biased(v, cb[qi], pos[qi] - (k0 + kt * 16 + 4 * g + e));
                        if (!inside && !seen(pos[qi], k0 + kt * 16 + 4 * g + e, W)) v = -INFINITY;
                        sc[qi][kt * 4 + e] = v;
                    }
            }
            v8bf w_hi[NQ], w_lo[NQ];
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) {
                if constexpr (SIGMOID) {
                    sigmoid_step(sc[qi], w_hi[qi], w_lo[qi]);
                } else {
                    const float fix = softmax_step(sc[qi], m[qi], l[qi], w_hi[qi], w_lo[qi]);
                    if (__any(fix != 1.0f)) {
#pragma unroll
                        for (int t = 0; t < VT; ++t) o[qi][t] *= fix;
                    }
                }
            }
#pragma unroll
            for (int t = 0; t < VT; ++t) {
                const v8bf v = transposed_keys(vb + t * 16, VP, lane);
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi) {
                    o[qi][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w_hi[qi], o[qi][t], 0, 0, 0);
                    o[qi][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w_lo[qi], o[qi][t], 0, 0, 0);
                }
            }
        }
        if (more) put(buf ^ 1);
        __syncthreads();
    }
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        float sum = SIGMOID ? 1.0f : l[qi];
        if constexpr (!SIGMOID) {
            sum += __shfl_xor(sum, 16, 64);
            sum += __shfl_xor(sum, 32, 64);
        }
        const uint32_t col = c0 + (wave * NQ + qi) * 16 + c;
        if (col >= n_cols) continue;
        const uint32_t head = kh * S + col % S;
        const float f = final_factor(ao, row0 + col / S, head, m[qi], sum);
        const OutputPlace at = output_place(out, ld_out, ao, sh, row0 + col / S, head);
#pragma unroll
        for (int t = 0; t < VT; ++t) store_columns(at, t * 16 + 4 * g, sh.vdim, o[qi][t] * f);
    }
}

// ------------------------------------------------------------------ which launches a pass needs
struct AttentionPlan {
    bool plain = false, stream = false, flash = false;
    uint32_t max_cols = 0;                           // columns of a sequence that is the few-rows kernel's
    int nq = 1;
    uint32_t tiles = 1, splits = 1;
};
AttentionPlan attention_plan(const AttentionShape &sh, const AttentionOutput &ao, int is_f32, uint32_t batch, uint32_t min_new, uint32_t max_new, uint32_t max_ctx, int num_cus) {
    AttentionPlan p;
    if (is_f32 || sh.dim_p > 256 || sh.v_p > 256 || g_attention_form == 1 || (ao.slope && !ao.sigmoid)) {
        p.plain = true;
        return p;
    }
    const uint32_t S = sh.share();
    p.max_cols = g_attention_form == 2 ? 0x7fffffffu : g_attention_form == 3 ? 0 : 64;
    p.stream = (uint64_t)min_new * S <= p.max_cols || (min_new <= 1 && p.max_cols);
    p.flash = (uint64_t)max_new * S > p.max_cols && (max_new > 1 || !p.max_cols);
    if (!p.stream) return p;
    // columns of the widest sequence the few-rows kernel may meet
    const uint64_t most = std::max<uint64_t>(S, std::min<uint64_t>((uint64_t)max_new * S, p.max_cols));
    p.nq = most <= 16 ? 1 : 2;
    p.tiles = (uint32_t)((most + 16 * p.nq - 1) / (16 * p.nq));
    const uint64_t blocks = (uint64_t)batch * ((uint64_t)(S * (uint64_t)std::max(1u, min_new) + 16 * p.nq - 1) / (16 * p.nq)) * sh.kv_heads;
    const uint64_t want = ((uint64_t)(g_attention_blocks ? g_attention_blocks : 1) * num_cus + blocks / 2) / std::max<uint64_t>(blocks, 1);
    const uint64_t span = std::min<uint64_t>(max_ctx, (uint64_t)sh.window + most / S);
    p.splits = (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({want, (span + 511) / 512, kMaxSplits}));
    return p;
}

constexpr int stream_waves(int d, int v) { return d == 8 || v == 8 ? 4 : 8; }

template <int D, int V, int NQ, bool SIGMOID>
void launch_stream(const StreamParams &p, const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    constexpr int NW = stream_waves(D, V);
    constexpr size_t stage = (size_t)NW * kKeys * (V * 32 + 8) * 2, meet = (size_t)NW / 2 * 16 * NQ * ((V * 32 + 4) * 4 + 8);
    constexpr size_t lds = stage > meet ? stage : meet;
    static_assert(lds <= 160 * 1024, "LDS of a compute unit");
    if constexpr (lds > 65536) {
        static bool configured = false;
        if (!configured) {
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&attention_stream_kernel<D, V, NQ, NW, SIGMOID>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            configured = true;
        }
    }
    attention_stream_kernel<D, V, NQ, NW, SIGMOID><<<dim3(rr.batch * p.tiles, sh.kv_heads, p.splits), NW * 64, lds, s>>>(p, sh, rr);
    if (p.splits > 1) attention_merge_kernel<<<dim3(rr.batch * p.tiles, sh.kv_heads, 16 * NQ), 64, 0, s>>>(p, sh, rr, 16 * NQ);
}

template <int D, int V, bool SIGMOID>
void launch_matrix_kind(const AttentionPlan &plan, const StreamParams &p, const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (plan.stream) {
        if (plan.nq == 1) launch_stream<D, V, 1, SIGMOID>(p, sh, rr, s);
        else launch_stream<D, V, 2, SIGMOID>(p, sh, rr, s);
    }
    if (plan.flash) {
        constexpr int NQ = D == 8 || V == 8 ? 1 : 2;
        constexpr size_t lds = 2ull * kKeys * (D * 32 + 8 + V * 32 + 8) * 2;
        if constexpr (lds > 65536) {
            static bool configured = false;
            if (!configured) {
                (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&attention_flash_kernel<D, V, NQ, SIGMOID>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
                configured = true;
            }
        }
        const dim3 grid((uint32_t)((uint64_t)rr.rows * sh.share() / (64 * NQ)) + rr.batch, sh.kv_heads);
        attention_flash_kernel<D, V, NQ, SIGMOID><<<grid, 256, lds, s>>>(p.q, p.k_pool, p.v_pool, p.out, p.ld_out, p.ao, plan.max_cols, sh, rr);
    }
}
template <int D, int V>
void launch_matrix(const AttentionPlan &plan, const StreamParams &p, const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (p.ao.sigmoid) launch_matrix_kind<D, V, true>(plan, p, sh, rr, s);
    else launch_matrix_kind<D, V, false>(plan, p, sh, rr, s);
}
template <int D>
void launch_matrix_v(const AttentionPlan &plan, const StreamParams &p, const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (sh.v_p == 64) launch_matrix<D, 2>(plan, p, sh, rr, s);
    else if (sh.v_p == 128) launch_matrix<D, 4>(plan, p, sh, rr, s);
    else launch_matrix<D, 8>(plan, p, sh, rr, s);
}

}  // namespace

void attention_pad(AttentionShape &sh) {
    auto up = [](uint32_t v) { return v <= 64 ? 64u : v <= 128 ? 128u : (v + 255) / 256 * 256; };
    sh.dim_p = up(sh.dim);
    sh.v_p = up(sh.vdim);
}

void attention_prepare(const float *y, uint32_t ld, const float *q_norm, const float *k_norm, void *q, void *k_pool, void *v_pool, int is_f32,
                       const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (rr.rows == 0) return;
    const bool vec = sh.dim % 4 == 0 && sh.vdim % 4 == 0 && ld % 4 == 0, wide = rr.rows <= 256 && sh.heads * sh.dim > 1024;
#define FA_PREP(T_, NT_, VEC_) \
    attention_prepare_kernel<T_, NT_, VEC_><<<rr.rows, NT_, 0, s>>>(y, ld, q_norm, k_norm, (T_ *)q, (T_ *)k_pool, (T_ *)v_pool, sh, rr.kv_slot)
    if (is_f32) {
        if (vec) FA_PREP(float, 256, true);
        else FA_PREP(float, 256, false);
    } else if (wide) {
        if (vec) FA_PREP(uint16_t, 1024, true);
        else FA_PREP(uint16_t, 1024, false);
    } else {
        if (vec) FA_PREP(uint16_t, 256, true);
        else FA_PREP(uint16_t, 256, false);
    }
#undef FA_PREP
}

void attention_prepare_heads(const float *y, uint32_t ld, bool norms, const float *q_norm, const float *k_norm, const float *cos_sin, bool key_values, void *q,
                             void *k_pool, void *v_pool, int is_f32, const AttentionShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (rr.rows == 0) return;
    const bool vec = sh.dim % 4 == 0 && sh.vdim % 4 == 0 && ld % 4 == 0 && sh.rot % (sh.interleaved ? 4 : 8) == 0;
    uint32_t group_log2 = 0;
    while (group_log2 < 6 && ((vec ? 4u : 1u) << group_log2) < sh.dim) ++group_log2;
    const PrepareHeads ph{q_norm, k_norm, cos_sin, norms, key_values};
    const uint32_t groups = 256u >> group_log2, units = sh.heads + 2 * sh.kv_heads;
    const dim3 grid(rr.rows, rr.rows <= 256 ? (units + groups - 1) / groups : 1);
#define FA_PREP(T_, VEC_) \
    attention_prepare_heads_kernel<T_, VEC_><<<grid, 256, 0, s>>>(y, ld, ph, (T_ *)q, (T_ *)k_pool, (T_ *)v_pool, sh, rr.kv_slot, rr.pos, group_log2)
    if (is_f32) {
        if (vec) FA_PREP(float, true);
        else FA_PREP(float, false);
    } else {
        if (vec) FA_PREP(uint16_t, true);
        else FA_PREP(uint16_t, false);
    }
#undef FA_PREP
}

uint64_t attention_workspace_bytes(const AttentionShape &sh, const AttentionOutput &ao, int is_f32, uint32_t batch, uint32_t min_new, uint32_t max_new, uint32_t max_ctx,
                                   int num_cus) {
    const AttentionPlan p = attention_plan(sh, ao, is_f32, batch, min_new, max_new, max_ctx, num_cus);
    return p.splits > 1 ? (uint64_t)batch * p.tiles * sh.kv_heads * p.splits * 16 * p.nq * (sh.v_p + 2) * 4 : 0;
}

void attention(const void *q, const void *k_pool, const void *v_pool, void *out, uint32_t ld_out, const AttentionOutput &ao, int is_f32,
               const AttentionShape &sh, const RaggedRows &rr, uint32_t min_new, uint32_t max_new, void *workspace, int num_cus, hipStream_t s) {
    if (rr.rows == 0) return;
    const AttentionPlan plan = attention_plan(sh, ao, is_f32, rr.batch, min_new, max_new, rr.max_blocks * rr.block_size, num_cus);
    if (plan.plain) {
        const dim3 grid(rr.rows, sh.heads);
        if (is_f32)
            attention_plain_kernel<float><<<grid, 256, sh.dim * 4, s>>>((const float *)q, (const float *)k_pool, (const float *)v_pool, (float *)out, ld_out, ao, sh, rr);
        else
            attention_plain_kernel<uint16_t><<<grid, 256, sh.dim * 4, s>>>((const uint16_t *)q, (const uint16_t *)k_pool, (const uint16_t *)v_pool,
                                                                           (uint16_t *)out, ld_out, ao, sh, rr);
        return;
    }
    StreamParams p{(const uint16_t *)q, (const uint16_t *)k_pool, (const uint16_t *)v_pool, (uint16_t *)out, ld_out, ao, (float *)workspace, nullptr, plan.splits,
                   plan.tiles, plan.max_cols};
    if (p.splits > 1) p.part_ml = p.part_o + (uint64_t)rr.batch * plan.tiles * sh.kv_heads * plan.splits * 16 * plan.nq * sh.v_p;
    if (sh.dim_p == 64) launch_matrix_v<2>(plan, p, sh, rr, s);
    else if (sh.dim_p == 128) launch_matrix_v<4>(plan, p, sh, rr, s);
    else launch_matrix_v<8>(plan, p, sh, rr, s);
}

}  // namespace k
}  // namespace fa
