// Linears on unquantized weights: bf16 on v_mfma_f32_16x16x32_bf16 (a weight-streaming kernel for up to 64 rows, a
// 128 x 128 tile kernel above that; kern_gemm_mfma.hip has the 256-row tiles for prompts), and a true f32 form for
// models that run in 32 bits.  All of them share the epilogues of LinearEpilogue.
// The matrix instruction takes the weight tile as its first operand, so lane l of an accumulator tile holds row
// l % 16 of the output and its columns 4 (l / 16) .. + 3.
#include <algorithm>

#include "device_utils.hpp"
#include "kernels.hpp"
#include "linear_epilogue.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_linear_form = 0;        // tuning: 2 keeps the large-tile kernel out, 3 four column tiles per block; grouped rows: 4 streamed
                              // weights, 5 128 x 128 tiles, 6 large tiles whatever the rows

namespace {

// ------------------------------------------------------------------ up to 64 rows
// A block owns NTW column tiles; its wavefronts take every NWAVES-th k tile, stream weights and activations through a
// ring of D register slots, and meet in LDS in a fixed order.  row_of(i): the activation row behind row i of the block's
// rows (i < m; others repeat row 0 and are never stored) and the output row.
template <int MT, int NTW, int NWAVES, int MODE, typename RowOf>
__device__ __forceinline__ void linear_rows(const uint16_t *__restrict__ a, uint64_t lda, const uint8_t *__restrict__ w_batch, uint32_t m,
                                            uint32_t n, uint32_t n_tiles, uint32_t k_tiles, uint32_t batch, const LinearEpilogue &ep, v4f *red_all,
                                            RowOf row_of) {
    static_assert(!is_glu(MODE) || NTW % 2 == 0, "gate and up are neighbouring tiles");
    constexpr int NT = MT * NTW, D = NTW == 4 || MT == 4 ? 4 : 8;
    v4f(*red)[NT][64] = (v4f(*)[NT][64])red_all;
    const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
    const uint32_t nt0 = blockIdx.x * NTW;
    const uint8_t *wb = w_batch + lane * 16;
    const uint8_t *a_row[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        uint32_t r = i * 16 + lane % 16;
        r = r < m ? r : 0;                       // a row past the end repeats row 0 and is never stored
        a_row[i] = (const uint8_t *)(a + (uint64_t)row_of(r).x * lda) + (lane / 16) * 16;
    }
    const uint32_t cnt = k_tiles > (uint32_t)wave ? (k_tiles - wave + NWAVES - 1) / NWAVES : 0;
    v4f acc[MT][NTW];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NTW; ++j) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};
    v4i av[D][MT], bv[D][NTW];
    auto load = [&](int s, uint32_t it) {
        const uint32_t kt = wave + (it < cnt ? it : cnt - 1) * NWAVES;
#pragma unroll
        for (int j = 0; j < NTW; ++j) {
            const uint32_t nt = nt0 + j < n_tiles ? nt0 + j : n_tiles - 1;
            bv[s][j] = stream_load<true>((const v4i *)(wb + ((uint64_t)nt * k_tiles + kt) * 1024));
        }
#pragma unroll
        for (int i = 0; i < MT; ++i) av[s][i] = *(const v4i *)(a_row[i] + (uint64_t)kt * 64);
    };
    auto mul = [&](int s) {
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
            for (int j = 0; j < NTW; ++j)
                acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(v8bf, bv[s][j]),
                                                                    __builtin_bit_cast(v8bf, av[s][i]), acc[i][j], 0, 0, 0);
    };
    if (cnt != 0) {
#pragma unroll
        for (int s = 0; s < D; ++s) load(s, (uint32_t)s);
        uint32_t it0 = 0;
        for (; it0 + D < cnt; it0 += D) {
#pragma unroll
            for (int s = 0; s < D; ++s) {
                mul(s);
                __builtin_amdgcn_sched_barrier(0);
                load(s, it0 + D + s);
                __builtin_amdgcn_sched_barrier(0);
            }
        }
#pragma unroll
        for (int s = 0; s < D; ++s)
            if (it0 + s < cnt) mul(s);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NTW; ++j) red[wave][i * NTW + j][lane] = acc[i][j];
    __syncthreads();
    auto total = [&](int t) {
        v4f r = red[0][t][lane];
#pragma unroll
        for (int q = 1; q < NWAVES; ++q) r += red[q][t][lane];
        return r;
    };
    constexpr int STEP = is_glu(MODE) ? 2 : 1;
    for (int t = wave * STEP; t < NT; t += NWAVES * STEP) {
        const int i = t / NTW, j = t % NTW;
        const uint32_t row = i * 16 + lane % 16;
        if (row >= m || nt0 + j >= n_tiles) continue;
        const v4f x = total(t);
        const v4f up = STEP == 2 ? total(t + 1) : x;
        const uint32_t tile = is_glu(MODE) ? (nt0 + j) / 2 : nt0 + j;
        epilogue_store4<MODE>(ep, row_of(row).y, tile * 16 + 4 * (lane / 16), n, batch, x, up);
    }
}

template <int MT, int NTW, int NWAVES, int MODE>
__global__ void __launch_bounds__(NWAVES * 64)
    linear_rows_kernel(const uint16_t *__restrict__ a, uint64_t lda, uint64_t a_batch, const uint8_t *__restrict__ w, uint32_t m,
                       uint32_t n, uint32_t n_tiles, uint32_t k_tiles, LinearEpilogue ep) {
    __shared__ v4f red[NWAVES * MT * NTW * 64];
    const uint32_t batch = blockIdx.y;
    linear_rows<MT, NTW, NWAVES, MODE>(a + batch * a_batch, lda, w + (uint64_t)batch * n_tiles * k_tiles * 1024, m, n, n_tiles, k_tiles, batch, ep, red,
                                       [](uint32_t r) { return make_uint2(r, r); });
}

// The rows of a group, up to 16 MT at a time (its weights then come from the caches again); groups without rows cost a
// launch slot only.
template <int MT, int NTW, int NWAVES, int MODE>
__global__ void __launch_bounds__(NWAVES * 64)
    linear_rows_grouped_kernel(const uint16_t *__restrict__ a, uint64_t lda, const uint8_t *__restrict__ w, uint32_t n, uint32_t n_tiles,
                               uint32_t k_tiles, RowGroups rg, LinearEpilogue ep) {
    __shared__ v4f red[NWAVES * MT * NTW * 64];
    const uint32_t group = blockIdx.y;
    uint32_t m = rg.count[group];
    m = m < rg.pitch ? m : rg.pitch;
    const uint8_t *wg = w + (uint64_t)group * n_tiles * k_tiles * 1024;
    for (uint32_t r0 = 0; r0 < m; r0 += 16 * MT) {
        const uint32_t left = m - r0;
        const uint32_t *list = rg.list + (uint64_t)group * rg.pitch + r0;
        auto row_of = [&](uint32_t r) {
            const uint32_t e = list[r];
            return make_uint2(e / rg.a_div, e);
        };
        if (r0) __syncthreads();
        if (MT == 1 || left <= 16) linear_rows<1, NTW, NWAVES, MODE>(a, lda, wg, left < 16 ? left : 16, n, n_tiles, k_tiles, 0, ep, red, row_of);
        else if (MT == 2 || left <= 32) linear_rows<(MT < 2 ? MT : 2), NTW, NWAVES, MODE>(a, lda, wg, left < 32 ? left : 32, n, n_tiles, k_tiles, 0, ep, red, row_of);
        else linear_rows<MT, NTW, NWAVES, MODE>(a, lda, wg, left < 16 * MT ? left : 16 * MT, n, n_tiles, k_tiles, 0, ep, red, row_of);
    }
}

// ------------------------------------------------------------------ 128 x 128 tiles
// Four wavefronts in 2 x 2, 64 x 64 each; a stage is two k tiles (64 values), double-buffered through registers.  LDS
// holds operand tiles in the instruction's lane order; the activation rows of k-group g are rotated by 4 g (+ 2 for the
// second k tile) so that the eight lanes that fetch one row's 128 bytes store to different banks.
template <int MODE, bool GROUPED = false>
__global__ void __launch_bounds__(256)
    linear_tile_kernel(const uint16_t *__restrict__ a, uint64_t lda, uint64_t a_batch, const uint8_t *__restrict__ w, uint32_t m,
                       uint32_t n, uint32_t n_tiles, uint32_t k_tiles, LinearEpilogue ep, RowGroups rg) {
    __shared__ __attribute__((aligned(16))) uint8_t lds_a[2][2][8 * 1024], lds_b[2][2][8 * 1024];   // [buffer][k tile]
    const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, wm = wave / 2, wn = wave % 2;
    uint32_t m0 = blockIdx.y * 128, nt0 = blockIdx.x * 8, batch = blockIdx.z;
    const uint32_t *list = nullptr;
    if constexpr (GROUPED) {
        uint32_t tile, column;
        if (!group_tile(rg, blockIdx.x, 128, (n_tiles + 7) / 8, &batch, &tile, &column)) return;
        m0 = tile * 128;
        nt0 = column * 8;
        m = rg.count[batch];
        list = rg.list + (uint64_t)batch * rg.pitch;
    }
    const uint8_t *ab = (const uint8_t *)(GROUPED ? a : a + batch * a_batch);
    const uint8_t *wb = w + (uint64_t)batch * n_tiles * k_tiles * 1024;
    uint32_t a_row[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint32_t row = m0 + threadIdx.x / 8 + 32 * i;
        a_row[i] = row < m ? row : m - 1;
        if constexpr (GROUPED) a_row[i] = list[a_row[i]] / rg.a_div;
    }
    v4u as[4], bs[4];
    const int piece = tid % 8, kt2 = piece / 4, kg = piece % 4;
    auto fetch = [&](uint32_t kt) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            as[i] = *(const v4u *)(ab + (uint64_t)a_row[i] * lda * 2 + (uint64_t)kt * 64 + piece * 16);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = tid + 256 * i;                 // 16-byte chunk of the stage: column tile c / 128, then k tile, then lane
            uint32_t nt = nt0 + c / 128;
            nt = nt < n_tiles ? nt : n_tiles - 1;
            bs[i] = *(const v4u *)(wb + ((uint64_t)nt * k_tiles + kt) * 1024 + (c % 128) * 16);
        }
    };
    auto put = [&](int buf) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = tid / 8 + 32 * i;
            *(v4u *)&lds_a[buf][kt2][(r / 16) * 1024 + (kg * 16 + ((r + 4 * kg + 2 * kt2) & 15)) * 16] = as[i];
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = tid + 256 * i;
            *(v4u *)&lds_b[buf][(c % 128) / 64][(c / 128) * 1024 + (c % 64) * 16] = bs[i];
        }
    };
    v4f acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = v4f{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    put(0);
    __syncthreads();
    for (uint32_t kt = 0; kt < k_tiles; kt += 2) {
        const int buf = (kt / 2) & 1;
        const bool more = kt + 2 < k_tiles;
        if (more) fetch(kt + 2);
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            v8bf av[4], bv[4];
            const int g = lane / 16, pos = (g * 16 + ((lane % 16 + 4 * g + 2 * h) & 15)) * 16;
#pragma unroll
            for (int i = 0; i < 4; ++i) av[i] = *(const v8bf *)&lds_a[buf][h][(wm * 4 + i) * 1024 + pos];
#pragma unroll
            for (int j = 0; j < 4; ++j) bv[j] = *(const v8bf *)&lds_b[buf][h][(wn * 4 + j) * 1024 + lane * 16];
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bv[j], av[i], acc[i][j], 0, 0, 0);
        }
        if (more) put(buf ^ 1);
        __syncthreads();
    }
    constexpr int STEP = is_glu(MODE) ? 2 : 1;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        uint32_t row = m0 + (wm * 4 + i) * 16 + lane % 16;
        if (row >= m) continue;
        if constexpr (GROUPED) row = list[row];
#pragma unroll
        for (int j = 0; j < 4; j += STEP) {
            const uint32_t nt = nt0 + wn * 4 + j;
            if (nt >= n_tiles) continue;
            const uint32_t tile = is_glu(MODE) ? nt / 2 : nt;
            epilogue_store4<MODE>(ep, row, tile * 16 + 4 * (lane / 16), n, GROUPED ? 0 : batch, acc[i][j], acc[i][j + STEP - 1]);
        }
    }
}

// ------------------------------------------------------------------ f32
// 64 x 64 outputs per block, 16 k per slab; thread (ty, tx) owns rows 4 ty .. + 3 of columns tx, tx + 16, tx + 32, tx + 48,
// so a gate column and its up column (the neighbouring tile of 16) sit in one thread.
template <int MODE, bool GROUPED = false>
__global__ void __launch_bounds__(256)
    linear_f32_kernel(const float *__restrict__ a, uint64_t lda, uint64_t a_batch, const float *__restrict__ w, uint32_t m, uint32_t n,
                      uint32_t n_tiles, uint32_t k_pad, LinearEpilogue ep, RowGroups rg) {
    __shared__ float as[16][68], bs[16][68];
    const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
    const uint32_t m0 = blockIdx.y * 64, n0 = blockIdx.x * 64, batch = blockIdx.z, n_rows = n_tiles * 16;
    const float *ab = GROUPED ? a : a + batch * a_batch, *wb = w + (uint64_t)batch * n_rows * k_pad;
    const uint32_t *list = nullptr;
    if constexpr (GROUPED) {
        m = rg.count[batch];
        list = rg.list + (uint64_t)batch * rg.pitch;
        if (m0 >= m) return;
    }
    const int r = tid / 4, c = (tid % 4) * 4;
    uint32_t ar = m0 + r < m ? m0 + r : m - 1;
    const uint32_t br = n0 + r < n_rows ? n0 + r : n_rows - 1;
    if constexpr (GROUPED) ar = list[ar] / rg.a_div;
    float acc[4][4] = {};
    for (uint32_t k0 = 0; k0 < k_pad; k0 += 16) {
        float va[4], vb[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            va[e] = ab[(uint64_t)ar * lda + k0 + c + e];
            vb[e] = wb[(uint64_t)br * k_pad + k0 + c + e];
        }
        __syncthreads();
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            as[c + e][r] = va[e];
            bs[c + e][r] = vb[e];
        }
        __syncthreads();
#pragma unroll
        for (int q = 0; q < 16; ++q)
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_fmaf(as[q][ty * 4 + i], bs[q][tx + 16 * j], acc[i][j]);
    }
    constexpr int STEP = is_glu(MODE) ? 2 : 1;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        uint32_t row = m0 + ty * 4 + i;
        if (row >= m) continue;
        if constexpr (GROUPED) row = list[row];
#pragma unroll
        for (int j = 0; j < 4; j += STEP) {
            const uint32_t nt = n0 / 16 + j;
            if (nt >= n_tiles) continue;
            const uint32_t col = (is_glu(MODE) ? nt / 2 : nt) * 16 + tx;
            if (col < n) epilogue_store1<MODE>(ep, row, col, GROUPED ? 0 : batch, acc[i][j], acc[i][j + STEP - 1]);
        }
    }
}

template <typename SRC, typename DST>
__global__ void __launch_bounds__(256)
    pack_linear_kernel(const SRC *__restrict__ src, uint64_t row_stride, uint64_t col_stride, uint32_t rows, uint32_t cols,
                       DST *__restrict__ dst, uint32_t k_tiles, uint32_t n0, uint32_t group, uint32_t pitch, uint32_t k0) {
    const uint64_t total = (uint64_t)rows * cols;
    for (uint64_t i = (uint64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (uint64_t)gridDim.x * 256) {
        const uint32_t r = (uint32_t)(i / cols), c = (uint32_t)(i % cols);
        const uint32_t nr = n0 + (r / group) * pitch + r % group;
        const SRC v = src[r * row_stride + c * col_stride];
        const uint32_t kc = k0 + c;
        if constexpr (sizeof(DST) == 4) {
            float f;
            if constexpr (sizeof(SRC) == 4) f = v;
            else f = bf16_to_f32(v);
            dst[(uint64_t)nr * k_tiles * 32 + kc] = f;
        } else {
            uint16_t h;
            if constexpr (sizeof(SRC) == 4) h = f32_to_bf16(v);
            else h = v;
            dst[((uint64_t)(nr / 16) * k_tiles + kc / 32) * 512 + (((kc % 32) / 8) * 16 + nr % 16) * 8 + kc % 8] = h;
        }
    }
}

template <int MODE>
void launch_bf16(const uint16_t *a, uint64_t lda, uint64_t a_batch, uint64_t m, const LinearWeight &w, const LinearEpilogue &ep,
                 int num_cus, hipStream_t s) {
    const uint8_t *wt = (const uint8_t *)w.w;
    if (m <= 64) {
        constexpr bool GLU = is_glu(MODE);
        const int mt = (int)((m + 15) / 16);
        // two tiles per block once one tile each would fill the device twice over; beyond 16 rows, where the registers allow
        // one block per compute unit, as soon as one tile each does not fit it at once
        const uint64_t tiles = (uint64_t)w.n_tiles * w.batches;
        const bool two = GLU || tiles >= 2 * (uint64_t)num_cus || (mt > 1 && tiles > (uint64_t)num_cus);
        // wide weights, up to 32 rows: four, so that the activations cross the L2 half as often
        const bool four = mt <= 2 && g_linear_form != 3 && w.batches == 1 && w.n_tiles >= 3 * (uint64_t)num_cus;
        const dim3 grid(four ? (w.n_tiles + 3) / 4 : two ? (w.n_tiles + 1) / 2 : w.n_tiles, w.batches);
#define FA_ROWS(MT_, NTW_)                                                                                             \
    linear_rows_kernel<MT_, NTW_, 8, MODE><<<grid, 512, 0, s>>>(a, lda, a_batch, wt, (uint32_t)m, w.n, w.n_tiles, w.k_tiles, ep)
        if (four) {
            if (mt == 1) FA_ROWS(1, 4);
            else FA_ROWS(2, 4);
        } else if constexpr (GLU) {
            if (mt == 1) FA_ROWS(1, 2);
            else if (mt == 2) FA_ROWS(2, 2);
            else FA_ROWS(4, 2);
        } else {
            if (mt == 1) two ? FA_ROWS(1, 2) : FA_ROWS(1, 1);
            else if (mt == 2) two ? FA_ROWS(2, 2) : FA_ROWS(2, 1);
            else two ? FA_ROWS(4, 2) : FA_ROWS(4, 1);
        }
#undef FA_ROWS
        return;
    }
    if (MODE != LinearEpilogue::kHeadGate && g_linear_form != 2 && gemm_bf16_big_applies(lda, m, w, ep, num_cus)) return gemm_bf16_big(a, m, w, ep, num_cus, s);
    const dim3 grid((w.n_tiles + 7) / 8, (unsigned)((m + 127) / 128), w.batches);
    linear_tile_kernel<MODE><<<grid, 256, 0, s>>>(a, lda, a_batch, wt, (uint32_t)m, w.n, w.n_tiles, w.k_tiles, ep, RowGroups{});
}

// Grouped rows: by the rows a group gets on average.  Few: weights streamed past them; a hundred and more: large tiles
// (16 experts of width 4096 and size 5376, 4 a token, passes of three layers, ms for 32 / 64 / 256 / 512 / 1024 rows: streamed 1.05 /
// 1.28 / 2.54 / 4.07 / 7.32, 128 x 128 tiles 1.13 / 1.20 / 1.54 / 1.92 / 2.87, large tiles 1.18 / 1.28 / 1.68 / 1.81 / 2.39).
template <int MODE>
void launch_grouped_bf16(const uint16_t *a, uint64_t lda, const LinearWeight &w, const RowGroups &rg, const LinearEpilogue &ep, int num_cus, hipStream_t s) {
    const uint8_t *wt = (const uint8_t *)w.w;
    constexpr bool GLU = is_glu(MODE);
    const uint64_t mean = (rg.likely ? rg.likely : rg.entries) / rg.groups;
    const int form = g_linear_form;
    if (form == 4 || (form != 5 && form != 6 && mean <= 10)) {
        const bool two = GLU || (uint64_t)w.n_tiles * std::min(rg.groups, rg.entries) >= 2 * (uint64_t)num_cus;
        const dim3 grid(two ? (w.n_tiles + 1) / 2 : w.n_tiles, rg.groups);
#define FA_ROWS(MT_, NTW_) linear_rows_grouped_kernel<MT_, NTW_, 8, MODE><<<grid, 512, 0, s>>>(a, lda, wt, w.n, w.n_tiles, w.k_tiles, rg, ep)
        if constexpr (GLU) {
            if (rg.most <= 16) FA_ROWS(1, 2);
            else if (mean <= 8) FA_ROWS(2, 2);
            else FA_ROWS(4, 2);
        } else {
            if (rg.most <= 16) two ? FA_ROWS(1, 2) : FA_ROWS(1, 1);
            else if (mean <= 8) two ? FA_ROWS(2, 2) : FA_ROWS(2, 1);
            else two ? FA_ROWS(4, 2) : FA_ROWS(4, 1);
        }
#undef FA_ROWS
        return;
    }
    if (form == 6 || (form != 5 && mean >= 112 && lda == (uint64_t)w.k_tiles * 32 && w.n_tiles >= 14)) return gemm_bf16_big_grouped(a, w, rg, ep, s);
    const uint32_t tiles = rg.entries / 128 + std::min(rg.groups, rg.entries);
    linear_tile_kernel<MODE, true><<<tiles * ((w.n_tiles + 7) / 8), 256, 0, s>>>(a, lda, 0, wt, 0, w.n, w.n_tiles, w.k_tiles, ep, rg);
}

template <int MODE>
void launch_grouped_f32(const float *a, uint64_t lda, const LinearWeight &w, const RowGroups &rg, const LinearEpilogue &ep, hipStream_t s) {
    const dim3 grid((w.n_tiles + 3) / 4, (unsigned)((rg.most + 63) / 64), rg.groups);
    linear_f32_kernel<MODE, true><<<grid, 256, 0, s>>>(a, lda, 0, (const float *)w.w, 0, w.n, w.n_tiles, w.k_tiles * 32, ep, rg);
}

template <int MODE>
void launch_f32(const float *a, uint64_t lda, uint64_t a_batch, uint64_t m, const LinearWeight &w, const LinearEpilogue &ep, hipStream_t s) {
    const dim3 grid((w.n_tiles + 3) / 4, (unsigned)((m + 63) / 64), w.batches);
    linear_f32_kernel<MODE><<<grid, 256, 0, s>>>(a, lda, a_batch, (const float *)w.w, (uint32_t)m, w.n, w.n_tiles, w.k_tiles * 32, ep, RowGroups{});
}

}  // namespace

void linear_bf16(const uint16_t *a, uint64_t lda, uint64_t a_batch, uint64_t m, const LinearWeight &w, const LinearEpilogue &ep,
                 int num_cus, hipStream_t s) {
    if (m == 0) return;
    switch (ep.mode) {
        case LinearEpilogue::kResidual: return launch_bf16<LinearEpilogue::kResidual>(a, lda, a_batch, m, w, ep, num_cus, s);
        case LinearEpilogue::kGlu: return launch_bf16<LinearEpilogue::kGlu>(a, lda, a_batch, m, w, ep, num_cus, s);
        case LinearEpilogue::kSiluGlu: return launch_bf16<LinearEpilogue::kSiluGlu>(a, lda, a_batch, m, w, ep, num_cus, s);
        case LinearEpilogue::kSoftcap: return launch_bf16<LinearEpilogue::kSoftcap>(a, lda, a_batch, m, w, ep, num_cus, s);
        case LinearEpilogue::kHeadGate: return launch_bf16<LinearEpilogue::kHeadGate>(a, lda, a_batch, m, w, ep, num_cus, s);
        case LinearEpilogue::kXielu: return launch_bf16<LinearEpilogue::kXielu>(a, lda, a_batch, m, w, ep, num_cus, s);
        default: return launch_bf16<LinearEpilogue::kStore>(a, lda, a_batch, m, w, ep, num_cus, s);
    }
}

void linear_f32(const float *a, uint64_t lda, uint64_t a_batch, uint64_t m, const LinearWeight &w, const LinearEpilogue &ep, hipStream_t s) {
    if (m == 0) return;
    switch (ep.mode) {
        case LinearEpilogue::kResidual: return launch_f32<LinearEpilogue::kResidual>(a, lda, a_batch, m, w, ep, s);
        case LinearEpilogue::kGlu: return launch_f32<LinearEpilogue::kGlu>(a, lda, a_batch, m, w, ep, s);
        case LinearEpilogue::kSiluGlu: return launch_f32<LinearEpilogue::kSiluGlu>(a, lda, a_batch, m, w, ep, s);
        case LinearEpilogue::kSoftcap: return launch_f32<LinearEpilogue::kSoftcap>(a, lda, a_batch, m, w, ep, s);
        case LinearEpilogue::kHeadGate: return launch_f32<LinearEpilogue::kHeadGate>(a, lda, a_batch, m, w, ep, s);
        case LinearEpilogue::kXielu: return launch_f32<LinearEpilogue::kXielu>(a, lda, a_batch, m, w, ep, s);
        default: return launch_f32<LinearEpilogue::kStore>(a, lda, a_batch, m, w, ep, s);
    }
}

void linear_grouped_bf16(const uint16_t *a, uint64_t lda, const LinearWeight &w, const RowGroups &rg, const LinearEpilogue &ep, int num_cus,
                         hipStream_t s) {
    if (rg.entries == 0 || rg.groups == 0) return;
    if (ep.mode == LinearEpilogue::kSquaredRelu) launch_grouped_bf16<LinearEpilogue::kSquaredRelu>(a, lda, w, rg, ep, num_cus, s);
    else if (ep.mode == LinearEpilogue::kSiluGlu) launch_grouped_bf16<LinearEpilogue::kSiluGlu>(a, lda, w, rg, ep, num_cus, s);
    else launch_grouped_bf16<LinearEpilogue::kStore>(a, lda, w, rg, ep, num_cus, s);
}

void linear_grouped_f32(const float *a, uint64_t lda, const LinearWeight &w, const RowGroups &rg, const LinearEpilogue &ep, hipStream_t s) {
    if (rg.entries == 0 || rg.groups == 0) return;
    if (ep.mode == LinearEpilogue::kSquaredRelu) launch_grouped_f32<LinearEpilogue::kSquaredRelu>(a, lda, w, rg, ep, s);
    else if (ep.mode == LinearEpilogue::kSiluGlu) launch_grouped_f32<LinearEpilogue::kSiluGlu>(a, lda, w, rg, ep, s);
    else launch_grouped_f32<LinearEpilogue::kStore>(a, lda, w, rg, ep, s);
}

void pack_linear(const void *src, int src_f32, uint64_t row_stride, uint64_t col_stride, uint32_t rows, uint32_t cols, void *dst,
                 int dst_f32, uint32_t k_tiles, uint32_t n0, uint32_t group, uint32_t pitch, hipStream_t s, uint32_t k0) {
    const uint64_t total = (uint64_t)rows * cols;
    if (total == 0) return;
    const unsigned grid = (unsigned)std::min<uint64_t>((total + 255) / 256, 8192);
    if (src_f32 && dst_f32)
        pack_linear_kernel<float, float><<<grid, 256, 0, s>>>((const float *)src, row_stride, col_stride, rows, cols, (float *)dst, k_tiles, n0, group, pitch, k0);
    else if (src_f32)
        pack_linear_kernel<float, uint16_t><<<grid, 256, 0, s>>>((const float *)src, row_stride, col_stride, rows, cols, (uint16_t *)dst, k_tiles, n0, group, pitch, k0);
    else if (dst_f32)
        pack_linear_kernel<uint16_t, float><<<grid, 256, 0, s>>>((const uint16_t *)src, row_stride, col_stride, rows, cols, (float *)dst, k_tiles, n0, group, pitch, k0);
    else
        pack_linear_kernel<uint16_t, uint16_t><<<grid, 256, 0, s>>>((const uint16_t *)src, row_stride, col_stride, rows, cols, (uint16_t *)dst, k_tiles, n0, group, pitch, k0);
}

}  // namespace k
}  // namespace fa
