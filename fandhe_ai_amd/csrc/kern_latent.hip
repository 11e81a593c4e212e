// Latent attention: queries and keys / values go through low-rank latents, and the cache holds, per token, only the normed
// latent and one rotated key part that all heads share.  The per-head key and value projections are absorbed into the
// query and the output, so every head attends to the same cached row [latent | rotated part] and sums latents.
#include <algorithm>
#include <type_traits>

#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_latent_form = 0;       // tuning: 1 keeps the plain attention kernel

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
        const float u = kr[i], v = kr[i + half];
        store_from_f32(dst + sh.rank_p + i, u * cs[i] - v * cs[half + i]);
        store_from_f32(dst + sh.rank_p + half + i, v * cs[i] + u * cs[half + i]);
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
            const float u = load_as_f32(src + d), v = load_as_f32(src + d + rh);
            store_from_f32(o + d, u * cs[d] - v * cs[rh + d]);
            store_from_f32(o + d + rh, v * cs[d] + u * cs[rh + d]);
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

uint64_t latent_attention_workspace_bytes(const LatentShape &sh, uint32_t rows, uint32_t batch) { return 0; }

void latent_attention(const void *qa, const void *pool, void *out, int is_f32, const LatentShape &sh, const RaggedRows &rr,
                      uint32_t max_new, void *workspace, int num_cus, hipStream_t s) {
    if (rr.rows == 0) return;
    const dim3 grid(rr.rows, sh.heads);
    const size_t lds = (size_t)(sh.rank_p + sh.rot_p) * 4;
    if (is_f32)
        latent_attention_plain_kernel<float><<<grid, 256, lds, s>>>((const float *)qa, (const float *)pool, (float *)out, sh, rr);
    else
        latent_attention_plain_kernel<uint16_t><<<grid, 256, lds, s>>>((const uint16_t *)qa, (const uint16_t *)pool, (uint16_t *)out, sh, rr);
}

}  // namespace k
}  // namespace fa
