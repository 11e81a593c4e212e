// Latent attention: queries and keys / values go through low-rank latents, and the cache holds, per token, only the normed
// latent and one rotated key part that all heads share.  The per-head key and value projections are absorbed into the
// query and the output, so every head attends to the same cached row [latent | rotated part] and sums latents.
#include <algorithm>
#include <type_traits>

#include "attention_tiles.hpp"
#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_latent_blocks = 0;     // tuning: blocks per compute unit the split of the keys aims at
int g_latent_form = 0;       // tuning: 1 keeps the plain attention kernel, 2 the absorbed form for every pass, 3 takes the
                             // expanded form wherever it can run

namespace {

// One block per row of y = q latent | kv latent | rotated key part | gates.
template <typename T>
__global__ void __launch_bounds__(256)
    latent_prepare_kernel(const float *__restrict__ y, uint32_t ld, const float *__restrict__ q_norm, const float *__restrict__ kv_norm,
                          const float *__restrict__ cos_sin, T *__restrict__ cq, uint32_t ld_cq, T *__restrict__ pool, LatentShape sh,
                          const uint32_t *__restrict__ kv_slot) {
    __shared__ float smem[4];
    const uint32_t r = blockIdx.x;
    const float *row = y + (uint64_t)r * ld;
    auto rms = [&](const float *v, uint32_t n) {
        float acc = 0.0f;
        for (uint32_t i = threadIdx.x; i < n; i += 256) acc = fmaf(v[i], v[i], acc);
        return 1.0f / sqrtf(block_sum<float, 4, true>(acc, smem) / (float)n + sh.eps);
    };
    const float rq = rms(row, sh.q_rank);
    for (uint32_t i = threadIdx.x; i < ld_cq; i += 256)
        store_from_f32(cq + (uint64_t)r * ld_cq + i, i < sh.q_rank ? row[i] * rq * q_norm[i] : 0.0f);
    if (!pool) return;                               // another layer's rows are used
    const float *c = row + sh.q_rank, *kr = c + sh.kv_rank;
    const float rc = rms(c, sh.kv_rank);
    const uint64_t slot = kv_slot[r];
    if (slot >= sh.pool_rows) return;
    T *dst = pool + slot * (sh.rank_p + sh.rot_p);
    for (uint32_t i = threadIdx.x; i < sh.kv_rank; i += 256) store_from_f32(dst + i, c[i] * rc * kv_norm[i]);
    const uint32_t half = sh.rot / 2;
    const float *cs = cos_sin + (uint64_t)r * sh.rot;
    for (uint32_t i = threadIdx.x; i < half; i += 256) {
        const uint2 at = rotation_pair(i, half, sh.interleaved);
        const float u = kr[at.x], v = kr[at.y];
        store_from_f32(dst + sh.rank_p + at.x, u * cs[i] - v * cs[half + i]);
        store_from_f32(dst + sh.rank_p + at.y, v * cs[i] + u * cs[half + i]);
    }
}

template <typename T>
__global__ void __launch_bounds__(256)
    latent_rotate_query_kernel(const T *__restrict__ q, const float *__restrict__ cos_sin, T *__restrict__ dst, uint32_t dst_pitch,
                               uint32_t dst_off, LatentShape sh) {
    const uint32_t r = blockIdx.x, half = sh.rot_p / 2, rh = sh.rot / 2;
    const float *cs = cos_sin + (uint64_t)r * sh.rot;
    for (uint32_t i = threadIdx.x; i < sh.heads * half; i += 256) {
        const uint32_t h = i / half, d = i % half;
        const T *src = q + ((uint64_t)r * sh.heads + h) * (sh.dim_p + sh.rot_p) + sh.dim_p;
        T *o = dst + ((uint64_t)r * sh.heads + h) * dst_pitch + dst_off;
        if (d < rh) {
            const uint2 at = rotation_pair(d, rh, sh.interleaved);
            const float u = load_as_f32(src + at.x), v = load_as_f32(src + at.y);
            store_from_f32(o + at.x, u * cs[d] - v * cs[rh + d]);
            store_from_f32(o + at.y, v * cs[d] + u * cs[rh + d]);
        } else {                                     // the padding behind the two halves
            store_from_f32(o + rh + d, 0.0f);
            store_from_f32(o + sh.rot_p - 1 - (d - rh), 0.0f);
        }
    }
}

// ------------------------------------------------------------------ plain form: any sizes, f32 or bf16
// One block per (row, head).  Keys are taken 256 at a time, one per thread for the scores, with a running maximum and sum;
// the threads then own latent dims.
constexpr uint32_t kPlainMaxRank = 2048;
template <typename T>
__global__ void __launch_bounds__(256)
    latent_attention_plain_kernel(const T *__restrict__ qa, const T *__restrict__ pool, T *__restrict__ out, LatentShape sh, RaggedRows rr) {
    extern __shared__ float lq[];                    // the query row
    __shared__ float w[256], smem[4];
    __shared__ uint32_t ids[256];
    const uint32_t r = blockIdx.x, h = blockIdx.y, width = sh.rank_p + sh.rot_p;
    const T *q = qa + ((uint64_t)r * sh.heads + h) * width;
    for (uint32_t i = threadIdx.x; i < width; i += 256) lq[i] = load_as_f32(q + i);
    const int32_t p = rr.pos[r];
    const uint32_t *table = rr.tables + (uint64_t)rr.row_seq[r] * rr.max_blocks;
    const int32_t first = p - (int32_t)sh.window + 1 > 0 ? p - (int32_t)sh.window + 1 : 0;
    float m = -INFINITY, l = 0.0f, acc[kPlainMaxRank / 256];
#pragma unroll
    for (uint32_t i = 0; i < kPlainMaxRank / 256; ++i) acc[i] = 0.0f;
    bool lost = false;                               // a position without a page: NaN, never a silent zero
    for (int32_t j0 = first; j0 <= p; j0 += 256) {
        __syncthreads();
        const int32_t j = j0 + (int32_t)threadIdx.x;
        float s = -INFINITY;
        uint32_t slot = 0;
        if (j <= p) {
            const uint32_t blk = (uint32_t)j / rr.block_size, id = blk < rr.max_blocks ? table[blk] : 0xffffffffu;
            if (id < rr.num_blocks) {
                slot = id * rr.block_size + (uint32_t)j % rr.block_size;
                const T *key = pool + (uint64_t)slot * width;
                float d = 0.0f;
                for (uint32_t i = 0; i < width; ++i) d = fmaf(lq[i], load_as_f32(key + i), d);
                s = d * sh.scale;
            } else {
                s = __uint_as_float(0x7fc00000u);
            }
        }
        ids[threadIdx.x] = slot;
        lost = lost || s != s;
        const float mc = fmaxf(m, block_max<4, true>(s, smem));
        const float e = j <= p ? expf(s - mc) : 0.0f, fix = expf(m - mc);
        w[threadIdx.x] = e;
        l = l * fix + block_sum<float, 4, true>(e, smem);        // its barriers publish w and ids
        m = mc;
        const int32_t n = p - j0 + 1 < 256 ? p - j0 + 1 : 256;
#pragma unroll
        for (uint32_t i = 0; i < kPlainMaxRank / 256; ++i) {
            const uint32_t d = threadIdx.x + i * 256;
            if (d >= sh.rank_p) continue;
            float a = acc[i] * fix;
            for (int32_t t = 0; t < n; ++t) a = fmaf(w[t], load_as_f32(pool + (uint64_t)ids[t] * width + d), a);
            acc[i] = a;
        }
    }
    if (__syncthreads_or(lost)) l = __uint_as_float(0x7fc00000u);
#pragma unroll
    for (uint32_t i = 0; i < kPlainMaxRank / 256; ++i) {
        const uint32_t d = threadIdx.x + i * 256;
        if (d < sh.rank_p) store_from_f32(out + ((uint64_t)r * sh.heads + h) * sh.rank_p + d, acc[i] / l);
    }
}

// ------------------------------------------------------------------ absorbed form
// Query rows of a sequence are its (token, head) pairs in order; a block takes NQ tiles of 16 of them, a tile being 16
// columns of S^T = K Q^T, and walks its share of the keys any of them sees, 32 at a time.  The cached rows of
// a step are staged once and serve as keys (all of the row) and, transposed, as values (the latent part).
// Block i of sequence b has slot row_start[b] heads / (16 NQ) + b + i: no two share one.
struct StreamParams {
    const uint16_t *qa, *pool;
    uint16_t *out;
    float *part_o, *part_ml;                         // [slot][split][16 NQ][rank_p], [slot][split][16 NQ][2]: maximum, sum
    uint32_t splits;
    int direct;                                      // one token per sequence, its heads in one block: block b is sequence b
};

template <int NQ>
__device__ __forceinline__ bool stream_tile(int direct, const RaggedRows &rr, uint32_t heads, uint32_t slot, uint32_t *b_out, uint32_t *t0, uint32_t *n_rows) {
    if (direct) {
        *b_out = slot;
        *t0 = 0;
        *n_rows = heads;
        return true;
    }
    auto base = [&](uint32_t b) { return (uint32_t)((uint64_t)rr.row_start[b] * heads / (16 * NQ)) + b; };
    uint32_t lo = 0, hi = rr.batch;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (base(mid) <= slot) lo = mid;
        else hi = mid;
    }
    *b_out = lo;
    *t0 = (slot - base(lo)) * 16 * NQ;
    *n_rows = (rr.row_start[lo + 1] - rr.row_start[lo]) * heads;
    return *t0 < *n_rows;
}

// RK, RO: rank_p and rot_p in units of 32.  DH wavefronts share a column tile: each forms the scores (registers for the
// whole query row) and sums a 1 / DH share of the latent dims.  GR groups of NQ DH wavefronts take a part of the block's keys
// each and meet in LDS at the end, which keeps partial results out of memory.
template <int RK, int RO, int NQ, int DH, int GR>
__global__ void __launch_bounds__(NQ * DH * GR * 64) __attribute__((amdgpu_waves_per_eu(2)))
    latent_stream_kernel(StreamParams p, LatentShape sh, RaggedRows rr) {
    constexpr int KS = RK + RO, VT = 2 * RK / DH, WIDTH = KS * 32, PITCH = WIDTH + 8, TPK = NQ * DH * 64 / kKeys;
    static_assert(VT % 4 == 0, "value tiles go in groups of four");
    constexpr int NP = (KS * 4 + TPK - 1) / TPK, KG = 2;
    extern __shared__ __attribute__((aligned(16))) uint16_t stage_all[];    // [GR][2][32][PITCH]
    uint32_t b, t0, n_rows;
    if (!stream_tile<NQ>(p.direct, rr, sh.heads, blockIdx.x, &b, &t0, &n_rows)) return;
    const int group = GR == 1 ? 0 : __builtin_amdgcn_readfirstlane(threadIdx.x / (NQ * DH * 64)), tid = threadIdx.x % (NQ * DH * 64);
    const int lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), qt = wave / DH, dh = wave % DH, g = lane / 16, c = lane % 16;
    uint16_t *stage = stage_all + group * 2 * kKeys * PITCH;
    const uint32_t row0 = rr.row_start[b], H = sh.heads;
    const uint32_t *table = rr.tables + (uint64_t)b * rr.max_blocks;
    const uint32_t last_row = t0 + 16 * NQ - 1 < n_rows ? t0 + 16 * NQ - 1 : n_rows - 1;
    const int32_t p0 = rr.pos[row0], p_lo = p0 + (int32_t)(t0 / H), p_hi = p0 + (int32_t)(last_row / H), W = (int32_t)sh.window;
    int32_t k_lo = p_lo - W + 1 > 0 ? p_lo - W + 1 : 0, k_hi = p_hi + 1;    // keys seen by some column
    if (p.splits > 1) {
        const int32_t per = ((k_hi - k_lo + (int32_t)p.splits - 1) / (int32_t)p.splits + kKeys - 1) / kKeys * kKeys;
        k_lo += (int32_t)blockIdx.y * per;
        k_hi = k_lo + per < k_hi ? k_lo + per : k_hi;
    }
    const uint64_t ps = ((uint64_t)blockIdx.x * p.splits + blockIdx.y) * 16 * NQ + qt * 16 + c;
    if (k_lo >= k_hi) {                              // a split without keys (never the only one)
        if (group == 0 && dh == 0 && g == 0) {
            p.part_ml[2 * ps] = -INFINITY;
            p.part_ml[2 * ps + 1] = 0.0f;
        }
        return;
    }
    const int32_t k_last = k_hi - 1;
    int32_t steps = (k_hi - k_lo + kKeys - 1) / kKeys;
    if (GR > 1) {                                    // this group's keys; every group runs the same number of steps
        steps = (steps + GR - 1) / GR;
        k_lo += group * steps * kKeys;
        k_hi = k_lo + steps * kKeys < k_hi ? k_lo + steps * kKeys : k_hi;
    }
    // staging: TPK threads per key, 16 bytes each at a time; keys past the walk repeat its last one (their weight is zero)
    const int key = tid / TPK, part = tid % TPK;
    v4u st[NP];
    bool lost = false;                               // the staged position has no page: NaN, never a silent zero
    auto page_of = [&](int32_t j) -> uint32_t {
        j = j <= k_last ? j : k_last;
        const uint32_t blk = (uint32_t)j / rr.block_size;
        return blk < rr.max_blocks ? table[blk] : 0xffffffffu;
    };
    auto fetch = [&](int32_t j, uint32_t id) {
        j = j <= k_last ? j : k_last;
        lost = id >= rr.num_blocks;
        const uint16_t *src = p.pool + ((uint64_t)(lost ? 0 : id) * rr.block_size + (uint32_t)j % rr.block_size) * WIDTH + part * 8;
#pragma unroll
        for (int i = 0; i < NP; ++i)
            if (NP * TPK == KS * 4 || part + i * TPK < KS * 4) st[i] = stream_load<true>((const v4u *)(src + i * TPK * 8));
    };
    auto put = [&](int buf) {
        if (lost) st[0] = v4u{0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u};
#pragma unroll
        for (int i = 0; i < NP; ++i)
            if (NP * TPK == KS * 4 || part + i * TPK < KS * 4) *(v4u *)(stage + (buf * kKeys + key) * PITCH + (part + i * TPK) * 8) = st[i];
    };
    uint32_t id = page_of(k_lo + key);
    uint32_t id_next = page_of(k_lo + kKeys + key);
    fetch(k_lo + key, id);
    // this lane's column
    const uint32_t col = t0 + qt * 16 + c, qr = col < n_rows ? col : n_rows - 1;
    const int32_t pos = p0 + (int32_t)(qr / H);
    const uint16_t *q = p.qa + ((uint64_t)row0 * H + qr) * WIDTH + 8 * g;
    v8bf qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) qf[s] = *(const v8bf *)(q + s * 32);
    hold(qf);
    const float factor = sh.scale * kLog2e;
    float m = -INFINITY, l = 0.0f;
    v4f o[VT];
#pragma unroll
    for (int t = 0; t < VT; ++t) o[t] = v4f{0.f, 0.f, 0.f, 0.f};
    put(0);
    __syncthreads();
    int buf = 0;
    for (int32_t it = 0, k0 = k_lo; it < steps; ++it, k0 += kKeys, buf ^= 1) {
        const bool more = it + 1 < steps;
        if (more) {
            fetch(k0 + kKeys + key, id_next);
            id_next = page_of(k0 + 2 * kKeys + key);
        }
        const uint16_t *rows = stage + buf * kKeys * PITCH;
        // operands are read a group ahead of the multiplies that take them
        v4f acc[2] = {v4f{0.f, 0.f, 0.f, 0.f}, v4f{0.f, 0.f, 0.f, 0.f}};
        v8bf kf[2][KG][2];
        auto read_keys = [&](int s0, v8bf (&d)[KG][2]) {
#pragma unroll
            for (int s = 0; s < KG; ++s)
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
                    if (s0 + s < KS) d[s][kt] = *(const v8bf *)(rows + (kt * 16 + c) * PITCH + (s0 + s) * 32 + 8 * g);
        };
        read_keys(0, kf[0]);
#pragma unroll
        for (int s0 = 0; s0 < KS; s0 += KG) {
            if (s0 + KG < KS) read_keys(s0 + KG, kf[(s0 / KG + 1) & 1]);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int s = 0; s < KG; ++s)
#pragma unroll
                for (int kt = 0; kt < 2; ++kt)
                    if (s0 + s < KS) acc[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[(s0 / KG) & 1][s][kt], qf[s0 + s], acc[kt], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
        float sc[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int32_t j = k0 + (i / 4) * 16 + 4 * g + i % 4;
            sc[i] = j <= pos && pos - j < W && j < k_hi ? acc[i / 4][i % 4] * factor : -INFINITY;
        }
        v8bf w_hi, w_lo;
        const float fix = softmax_step(sc, m, l, w_hi, w_lo);
        if (__any(fix != 1.0f)) {
#pragma unroll
            for (int t = 0; t < VT; ++t) o[t] *= fix;
        }
        v8bf vf[2][4];
#pragma unroll
        for (int i = 0; i < 4; ++i) vf[0][i] = transposed_keys(rows + (dh * VT + i) * 16, PITCH, lane);
#pragma unroll
        for (int t = 0; t < VT; t += 4) {
            if (t + 4 < VT) {
#pragma unroll
                for (int i = 0; i < 4; ++i) vf[(t / 4 + 1) & 1][i] = transposed_keys(rows + (dh * VT + t + 4 + i) * 16, PITCH, lane);
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int i = 0; i < 4; ++i) o[t + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[(t / 4) & 1][i], w_hi, o[t + i], 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; ++i) o[t + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[(t / 4) & 1][i], w_lo, o[t + i], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
        if (more) put(buf ^ 1);
        __syncthreads();
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if constexpr (GR == 2) {
        constexpr int OP = RK * 32 + 4;              // pitch of an exchanged row
        static_assert(16 * NQ * (OP * 4 + 8) <= GR * 2 * kKeys * PITCH * 2, "the exchange fits the stages");
        float *xo = (float *)stage_all, *xm = xo + 16 * NQ * OP;
        if (group == 1) {
            if (g == 0) {
                xm[(qt * 16 + c) * 2] = m;
                xm[(qt * 16 + c) * 2 + 1] = l;
            }
#pragma unroll
            for (int t = 0; t < VT; ++t) *(v4f *)(xo + (qt * 16 + c) * OP + (dh * VT + t) * 16 + 4 * g) = o[t];
        }
        __syncthreads();
        if (group == 1) return;
        const float m1 = xm[(qt * 16 + c) * 2], l1 = xm[(qt * 16 + c) * 2 + 1], mx = fmaxf(m, m1), ref = mx == -INFINITY ? 0.0f : mx;
        const float f0 = exp2f(m - ref), f1 = exp2f(m1 - ref);
        m = mx;
        l = l * f0 + l1 * f1;
#pragma unroll
        for (int t = 0; t < VT; ++t) o[t] = o[t] * f0 + *(const v4f *)(xo + (qt * 16 + c) * OP + (dh * VT + t) * 16 + 4 * g) * f1;
    }
    if (p.splits > 1) {
        if (dh == 0 && g == 0) {
            p.part_ml[2 * ps] = m;
            p.part_ml[2 * ps + 1] = l;
        }
        if (col < n_rows) {
#pragma unroll
            for (int t = 0; t < VT; ++t) *(v4f *)(p.part_o + ps * (RK * 32) + (dh * VT + t) * 16 + 4 * g) = o[t];
        }
        return;
    }
    if (col >= n_rows) return;
    const float inv = 1.0f / l;
#pragma unroll
    for (int t = 0; t < VT; ++t)
        *(v2u *)(p.out + ((uint64_t)row0 * H + col) * (RK * 32) + (dh * VT + t) * 16 + 4 * g) =
            v2u{f32x2_to_bf16x2(o[t][0] * inv, o[t][1] * inv), f32x2_to_bf16x2(o[t][2] * inv, o[t][3] * inv)};
}

// Adds the splits of a tile's columns: one block per (slot, column), four dims per thread.
constexpr uint32_t kMaxSplits = 64;
template <int NQ>
__global__ void __launch_bounds__(128) latent_merge_kernel(StreamParams p, LatentShape sh, RaggedRows rr) {
    __shared__ float w[kMaxSplits];
    uint32_t b, t0, n_rows;
    if (!stream_tile<NQ>(p.direct, rr, sh.heads, blockIdx.x, &b, &t0, &n_rows)) return;
    const uint32_t cl = blockIdx.y, col = t0 + cl;
    if (col >= n_rows) return;
    const uint64_t ps = (uint64_t)blockIdx.x * p.splits * 16 * NQ + cl;      // split s of this column: + s * 16 NQ
    if (threadIdx.x < 64) {
        const uint32_t s = threadIdx.x;
        float ms = -INFINITY, ls = 0.0f;                                     // sum 0: the split holds none of the column's keys
        if (s < p.splits) {
            const v2f v = *(const v2f *)(p.part_ml + 2 * (ps + (uint64_t)s * 16 * NQ));
            ms = v[0];
            ls = v[1];
        }
        const float m = wave_max(ms), f = ls != 0.0f ? exp2f(ms - m) : 0.0f, l = wave_sum(ls * f);
        w[s] = f / l;
    }
    __syncthreads();
    for (uint32_t d = threadIdx.x * 4; d < sh.rank_p; d += 512) {
        const float *src = p.part_o + ps * sh.rank_p + d;
        v4f a = v4f{0.f, 0.f, 0.f, 0.f};
        for (uint32_t s0 = 0; s0 < p.splits; s0 += 8) {
            v4f t[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) t[i] = *(const v4f *)(src + (uint64_t)(s0 + i < p.splits ? s0 + i : p.splits - 1) * 16 * NQ * sh.rank_p);
#pragma unroll
            for (int i = 0; i < 8; ++i)
                if (s0 + i < p.splits && w[s0 + i] != 0.0f) a += t[i] * w[s0 + i];
        }
        *(v2u *)(p.out + ((uint64_t)rr.row_start[b] * sh.heads + col) * sh.rank_p + d) = v2u{f32x2_to_bf16x2(a[0], a[1]), f32x2_to_bf16x2(a[2], a[3])};
    }
}

// Key groups of a block: two for the few query rows of a decode step
constexpr int stream_groups(int nq) { return nq == 2 ? 2 : 1; }

struct StreamPlan {
    int nq = 0, direct = 0;                          // nq 0: the plain kernel
    uint32_t slots = 0, splits = 1;
};
StreamPlan stream_plan(const LatentShape &sh, uint32_t rows, uint32_t batch, uint32_t longest, int num_cus) {
    StreamPlan p;
    if (sh.rank_p > 512 || sh.rot_p > 64 || g_latent_form == 1) return p;
    p.nq = (uint64_t)longest * sh.heads <= 32 ? 2 : 4;
    p.direct = longest == 1 && rows == batch && sh.heads <= 16u * p.nq;
    p.slots = p.direct ? batch : (uint32_t)((uint64_t)rows * sh.heads / (16 * p.nq)) + batch + 1;
    // wavefronts for about two blocks of one key group per compute unit, at least 128 keys each; the number of used slots is close to rows * heads / (16 NQ)
    const uint64_t used = std::max<uint64_t>(std::max<uint64_t>((uint64_t)rows * sh.heads / (16 * p.nq), batch), 1);
    const uint64_t per_cu = g_latent_blocks ? g_latent_blocks : 3 - stream_groups(p.nq), least = 128 * stream_groups(p.nq);
    const uint64_t want = (per_cu * num_cus + used - 1) / used;
    p.splits = (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({want, (sh.window + least - 1) / least, kMaxSplits}));
    return p;
}

template <int RK, int RO, int NQ>
void launch_stream(const StreamParams &p, const LatentShape &sh, const RaggedRows &rr, uint32_t slots, hipStream_t s) {
    constexpr int DH = RK == 16 ? 2 : 1, GR = stream_groups(NQ);
    constexpr size_t lds = GR * 2ull * kKeys * ((RK + RO) * 32 + 8) * 2;
    if constexpr (lds > 65536) {
        static bool configured = false;
        if (!configured) {
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_stream_kernel<RK, RO, NQ, DH, GR>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            configured = true;
        }
    }
    latent_stream_kernel<RK, RO, NQ, DH, GR><<<dim3(slots, p.splits), NQ * DH * GR * 64, lds, s>>>(p, sh, rr);
    if (p.splits > 1) latent_merge_kernel<NQ><<<dim3(slots, 16 * NQ), 128, 0, s>>>(p, sh, rr);
}
template <int RK, int RO>
void launch_stream_nq(const StreamParams &p, const LatentShape &sh, const RaggedRows &rr, const StreamPlan &plan, hipStream_t s) {
    if (plan.nq == 2) launch_stream<RK, RO, 2>(p, sh, rr, plan.slots, s);
    else launch_stream<RK, RO, 4>(p, sh, rr, plan.slots, s);
}
template <int RK>
void launch_stream_ro(const StreamParams &p, const LatentShape &sh, const RaggedRows &rr, const StreamPlan &plan, hipStream_t s) {
    if (sh.rot_p <= 32) launch_stream_nq<RK, 1>(p, sh, rr, plan, s);
    else launch_stream_nq<RK, 2>(p, sh, rr, plan, s);
}

// ------------------------------------------------------------------ expanded form
// Prompts: the keys and values of every cached token the pass sees are formed per head (one linear), and attention runs per
// head on them: per query and key 2 (dim + rot + vdim) operations instead of 2 (2 rank + rot).
__global__ void __launch_bounds__(256)
    latent_gather_kernel(const uint16_t *__restrict__ pool, uint16_t *__restrict__ c, uint32_t ld_c, uint16_t *__restrict__ kr, LatentShape sh,
                         RaggedRows rr, LatentExpand ex) {
    const uint32_t e = blockIdx.x * 4 + threadIdx.x / 64, lane = threadIdx.x % 64;
    if (e >= ex.rows) return;
    uint32_t lo = 0, hi = rr.batch;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (ex.start[mid] <= e) lo = mid;
        else hi = mid;
    }
    const uint32_t j = ex.first[lo] + (e - ex.start[lo]), width = sh.rank_p + sh.rot_p, blk = j / rr.block_size;
    const uint32_t id = blk < rr.max_blocks ? rr.tables[(uint64_t)lo * rr.max_blocks + blk] : 0xffffffffu;
    const bool ok = id < rr.num_blocks;
    const uint16_t *src = pool + ((uint64_t)(ok ? id : 0) * rr.block_size + j % rr.block_size) * width;
    for (uint32_t i = lane * 8; i < ld_c + sh.rot_p; i += 512) {
        v4u v = ok ? v4u{0, 0, 0, 0} : v4u{0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u};
        if (i < ld_c) {
            if (ok && i < sh.rank_p) v = *(const v4u *)(src + i);
            *(v4u *)(c + (uint64_t)e * ld_c + i) = v;
        } else {
            if (ok) v = *(const v4u *)(src + sh.rank_p + (i - ld_c));
            *(v4u *)(kr + (uint64_t)e * sh.rot_p + (i - ld_c)) = v;
        }
    }
}

// A block of four wavefronts takes 128 tokens of one (sequence, head), every wavefront 32 columns of S^T = K Q^T, and walks
// the keys they see 32 at a time; K (unrotated | rotated) and V of a step are staged in LDS, two stages.  D, RO:
// dim_p = v_p and rot_p in units of 32.
template <int D, int RO>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 2)))
    latent_flash_kernel(const uint16_t *__restrict__ q, const uint16_t *__restrict__ kv, const uint16_t *__restrict__ kr,
                        const float *__restrict__ gate, uint32_t ld_gate, float out_scale, uint16_t *__restrict__ out, uint32_t ld_out,
                        LatentShape sh, RaggedRows rr, LatentExpand ex) {
    constexpr int KS = D + RO, VT = 2 * D, KP = KS * 32 + 8, VP = D * 32 + 8, NQ = 2;
    constexpr int PKR = (KS * 4 + 7) / 8, PV = D * 4 / 8;        // 16-byte pieces per thread and step, eight threads per key
    __shared__ __attribute__((aligned(16))) uint16_t ks[2][kKeys * KP], vs[2][kKeys * VP];
    // longest walks first: the last tiles of a sequence
    uint32_t lo = 0, hi = rr.batch;
    const uint32_t slots = gridDim.x, slot = slots - 1 - blockIdx.x;
    while (hi - lo > 1) {
        const uint32_t mid = (lo + hi) / 2;
        if (rr.row_start[mid] / 128 + mid <= slot) lo = mid;
        else hi = mid;
    }
    const uint32_t b = lo, row0 = rr.row_start[b], n = rr.row_start[b + 1] - row0, t0 = (slot - (row0 / 128 + b)) * 128;
    if (t0 >= n) return;
    const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), g = lane / 16, c = lane % 16;
    const uint32_t h = blockIdx.y, H = sh.heads, qw = KS * 32;
    constexpr uint32_t hw = 2 * D * 32;              // one head of an expanded row
    const int32_t p0 = rr.pos[row0], W = (int32_t)sh.window, first = (int32_t)ex.first[b];
    const uint32_t t_last = t0 + 127 < n ? t0 + 127 : n - 1;
    int32_t k_lo = p0 + (int32_t)t0 - W + 1, k_hi = p0 + (int32_t)t_last + 1;
    k_lo = k_lo > first ? k_lo : first;
    const uint64_t e0 = (uint64_t)ex.start[b] - (uint64_t)first;     // expanded row of key j: e0 + j

    v8bf qf[NQ][KS];
    int32_t pos[NQ];
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        uint32_t t = t0 + wave * 32 + qi * 16 + c;
        t = t < n ? t : n - 1;
        pos[qi] = p0 + (int32_t)t;
        const uint16_t *src = q + ((uint64_t)(row0 + t) * H + h) * qw + 8 * g;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            qf[qi][s] = *(const v8bf *)(src + s * 32);
        }
    }
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) hold(qf[qi]);
    const int32_t w_lo_pos = p0 + (int32_t)(t0 + wave * 32 < n ? t0 + wave * 32 : n - 1);
    const int32_t w_hi_pos = p0 + (int32_t)(t0 + wave * 32 + 31 < n ? t0 + wave * 32 + 31 : n - 1);

    const int key = tid / 8, part = tid % 8;
    v4u sk[PKR], sv[PV];
    auto fetch = [&](int32_t k0) {
        const int32_t j = k0 + key;
        const bool ok = j < k_hi;
        const uint64_t e = e0 + (uint64_t)(ok ? j : k_hi - 1);
        const uint16_t *row = kv + (e * H + h) * hw, *rot = kr + e * (RO * 32);
#pragma unroll
        for (int i = 0; i < PKR; ++i) {
            const int pc = part + 8 * i;
            if (pc < KS * 4) sk[i] = *(const v4u *)(pc < D * 4 ? row + pc * 8 : rot + (pc - D * 4) * 8);
        }
#pragma unroll
        for (int i = 0; i < PV; ++i) sv[i] = *(const v4u *)(row + D * 32 + (part + 8 * i) * 8);
    };
    auto put = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PKR; ++i)
            if (part + 8 * i < KS * 4) *(v4u *)&ks[buf][key * KP + (part + 8 * i) * 8] = sk[i];
#pragma unroll
        for (int i = 0; i < PV; ++i) *(v4u *)&vs[buf][key * VP + (part + 8 * i) * 8] = sv[i];
    };
    float m[NQ], l[NQ];
    v4f o[NQ][VT];
#pragma unroll
    for (int qi = 0; qi < NQ; ++qi) {
        m[qi] = -INFINITY;
        l[qi] = 0.0f;
#pragma unroll
        for (int t = 0; t < VT; ++t) o[qi][t] = v4f{0.f, 0.f, 0.f, 0.f};
    }
    fetch(k_lo);
    put(0);
    __syncthreads();
    int buf = 0;
    for (int32_t k0 = k_lo; k0 < k_hi; k0 += kKeys, buf ^= 1) {
        const bool more = k0 + kKeys < k_hi;
        if (more) fetch(k0 + kKeys);
        if (k0 <= w_hi_pos && k0 + kKeys > w_lo_pos - W + 1) {       // some column of this wavefront sees some key of the step
            const bool inside = k0 + kKeys - 1 <= w_lo_pos && k0 > w_hi_pos - W;       // every column sees every key
            float sc[NQ][8];
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                v4f acc[NQ];
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi) acc[qi] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < KS; ++s) {
                    const v8bf kf = *(const v8bf *)&ks[buf][(kt * 16 + c) * KP + s * 32 + 8 * g];
#pragma unroll
                    for (int qi = 0; qi < NQ; ++qi) acc[qi] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qi][s], acc[qi], 0, 0, 0);
                }
#pragma unroll
                for (int qi = 0; qi < NQ; ++qi)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        float v = acc[qi][e] * (sh.scale * kLog2e);
                        if (!inside) {
                            const int32_t j = k0 + kt * 16 + 4 * g + e;
                            if (j > pos[qi] || pos[qi] - j >= W) v = -INFINITY;
                        }
                        sc[qi][kt * 4 + e] = v;
                    }
            }
            v8bf w_hi[NQ], w_lo[NQ];
#pragma unroll
            for (int qi = 0; qi < NQ; ++qi) {
                const float fix = softmax_step(sc[qi], m[qi], l[qi], w_hi[qi], w_lo[qi]);
                if (__any(fix != 1.0f)) {
#pragma unroll
                    for (int t = 0; t < VT; ++t) o[qi][t] *= fix;
                }
            }
#pragma unroll
            for (int t = 0; t < VT; ++t) {
                const v8bf v = transposed_keys(&vs[buf][t * 16], VP, lane);
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
        float sum = l[qi];
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        const uint32_t t = t0 + wave * 32 + qi * 16 + c;
        if (t >= n) continue;
        const float f = gate ? out_scale / (1.0f + expf(-gate[(uint64_t)(row0 + t) * ld_gate + h])) / sum : out_scale / sum;
        uint16_t *dst = out + (uint64_t)(row0 + t) * ld_out + h * sh.vdim;
        const bool vec = (sh.vdim & 3) == 0;
#pragma unroll
        for (int dt = 0; dt < VT; ++dt) {
            const uint32_t d = dt * 16 + 4 * g;
            if (vec && d < sh.vdim)
                *(v2u *)(dst + d) = v2u{f32x2_to_bf16x2(o[qi][dt][0] * f, o[qi][dt][1] * f), f32x2_to_bf16x2(o[qi][dt][2] * f, o[qi][dt][3] * f)};
            else if (!vec) {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (d + e < sh.vdim) dst[d + e] = f32_to_bf16(o[qi][dt][e] * f);
            }
        }
    }
}

}  // namespace

void latent_prepare(const float *y, uint32_t ld, const float *q_norm, const float *kv_norm, const float *cos_sin, void *cq,
                    uint32_t ld_cq, void *pool, int is_f32, const LatentShape &sh, const RaggedRows &rr, hipStream_t s) {
    if (rr.rows == 0) return;
    if (is_f32)
        latent_prepare_kernel<float><<<rr.rows, 256, 0, s>>>(y, ld, q_norm, kv_norm, cos_sin, (float *)cq, ld_cq, (float *)pool, sh, rr.kv_slot);
    else
        latent_prepare_kernel<uint16_t><<<rr.rows, 256, 0, s>>>(y, ld, q_norm, kv_norm, cos_sin, (uint16_t *)cq, ld_cq, (uint16_t *)pool, sh, rr.kv_slot);
}

void latent_rotate_query(const void *q, const float *cos_sin, void *dst, uint32_t dst_pitch, uint32_t dst_off, int is_f32,
                         const LatentShape &sh, uint32_t rows, hipStream_t s) {
    if (rows == 0) return;
    if (is_f32)
        latent_rotate_query_kernel<float><<<rows, 256, 0, s>>>((const float *)q, cos_sin, (float *)dst, dst_pitch, dst_off, sh);
    else
        latent_rotate_query_kernel<uint16_t><<<rows, 256, 0, s>>>((const uint16_t *)q, cos_sin, (uint16_t *)dst, dst_pitch, dst_off, sh);
}

void latent_pad(LatentShape &sh) {
    auto up = [](uint32_t v, std::initializer_list<uint32_t> sizes) {
        for (uint32_t s : sizes)
            if (v <= s) return s;
        return (v + 31) / 32 * 32;
    };
    sh.rank_p = up(sh.kv_rank, {64, 128, 256, 512});
    sh.rot_p = up(sh.rot, {32, 64});
    sh.dim_p = up(sh.dim, {64, 128});
    sh.v_p = up(sh.vdim, {64, 128});
    if (sh.dim_p <= 128 && sh.v_p <= 128) sh.dim_p = sh.v_p = sh.dim_p > sh.v_p ? sh.dim_p : sh.v_p;
}

uint64_t latent_attention_workspace_bytes(const LatentShape &sh, int is_f32, uint32_t rows, uint32_t batch, uint32_t max_new, int num_cus) {
    if (is_f32) return 0;
    const StreamPlan p = stream_plan(sh, rows, batch, max_new, num_cus);
    return p.splits > 1 ? (uint64_t)p.slots * p.splits * 16 * p.nq * (sh.rank_p + 2) * 4 : 0;
}

void latent_attention(const void *qa, const void *pool, void *out, int is_f32, const LatentShape &sh, const RaggedRows &rr,
                      uint32_t max_new, void *workspace, int num_cus, hipStream_t s) {
    if (rr.rows == 0) return;
    if (!is_f32) {
        const StreamPlan plan = stream_plan(sh, rr.rows, rr.batch, max_new, num_cus);
        if (plan.nq) {
            StreamParams p{(const uint16_t *)qa, (const uint16_t *)pool, (uint16_t *)out, (float *)workspace, nullptr, plan.splits, plan.direct};
            if (p.splits > 1) p.part_ml = p.part_o + (uint64_t)plan.slots * plan.splits * 16 * plan.nq * sh.rank_p;
            if (sh.rank_p <= 64) launch_stream_ro<2>(p, sh, rr, plan, s);
            else if (sh.rank_p <= 128) launch_stream_ro<4>(p, sh, rr, plan, s);
            else if (sh.rank_p <= 256) launch_stream_ro<8>(p, sh, rr, plan, s);
            else launch_stream_ro<16>(p, sh, rr, plan, s);
            return;
        }
    }
    const dim3 grid(rr.rows, sh.heads);
    const size_t lds = (size_t)(sh.rank_p + sh.rot_p) * 4;
    if (is_f32)
        latent_attention_plain_kernel<float><<<grid, 256, lds, s>>>((const float *)qa, (const float *)pool, (float *)out, sh, rr);
    else
        latent_attention_plain_kernel<uint16_t><<<grid, 256, lds, s>>>((const uint16_t *)qa, (const uint16_t *)pool, (uint16_t *)out, sh, rr);
}

bool latent_expand_applies(const LatentShape &sh) {
    return sh.dim_p == sh.v_p && sh.v_p <= 128 && sh.rot_p <= 64 && g_latent_form != 1 && g_latent_form != 2;
}
bool latent_expand_always() { return g_latent_form == 3; }

void latent_gather(const void *pool, void *c, uint32_t ld_c, void *kr, const LatentShape &sh, const RaggedRows &rr, const LatentExpand &ex, hipStream_t s) {
    if (ex.rows == 0) return;
    latent_gather_kernel<<<(ex.rows + 3) / 4, 256, 0, s>>>((const uint16_t *)pool, (uint16_t *)c, ld_c, (uint16_t *)kr, sh, rr, ex);
}

void latent_attention_expanded(const void *q, const void *kv, const void *kr, const float *gate, uint32_t ld_gate, float out_scale, void *out,
                               uint32_t ld_out, const LatentShape &sh, const RaggedRows &rr, const LatentExpand &ex, hipStream_t s) {
    const dim3 grid(rr.rows / 128 + rr.batch + 1, sh.heads);
    const bool wide = sh.v_p > 64, rot2 = sh.rot_p > 32;
#define FA_FLASH(D_, RO_)                                                                                                                    \
    latent_flash_kernel<D_, RO_><<<grid, 256, 0, s>>>((const uint16_t *)q, (const uint16_t *)kv, (const uint16_t *)kr, gate, ld_gate, out_scale, \
                                                      (uint16_t *)out, ld_out, sh, rr, ex)
    if (wide) rot2 ? FA_FLASH(4, 2) : FA_FLASH(4, 1);
    else rot2 ? FA_FLASH(2, 2) : FA_FLASH(2, 1);
#undef FA_FLASH
}

}  // namespace k
}  // namespace fa
