// Residual updates with the norms around them, and the routing of sparse feed-forwards: the weighted sum of a row's experts, the
// router with the choice of experts.  The experts' linears are kern_linear.hip's.
#include <algorithm>

#include "attention_tiles.hpp"
#include "device_utils.hpp"
#include "kernels.hpp"

namespace fa {
namespace k {
using namespace fa::dev;

int g_route_form = 0;         // tuning: 1 the router in the residual update whatever the rows, 2 in a launch of its own

namespace {

// The largest value of a row that is not taken yet (ties: the lower index), by one wavefront: value i of lane l is the row's
// 64 i + l, bit i of `taken` says that it is out.  It is taken; false where none is left.
template <int N>
__device__ __forceinline__ bool take_largest(const float (&v)[N], uint32_t &taken, int lane, uint32_t *index, float *value) {
    float best = -INFINITY;
#pragma unroll
    for (int i = 0; i < N; ++i)
        if (!(taken >> i & 1)) best = fmaxf(best, v[i]);
    best = wave_max_dpp(best);
    *value = best;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint64_t there = __ballot(!(taken >> i & 1) && v[i] == best);
        if (there) {
            const int at = __builtin_ctzll(there);
            *index = i * 64 + at;
            if (lane == at) taken |= 1u << i;
            return true;
        }
    }
    return false;
}

// The experts of one row from its logits (LDS), by one wavefront: lane i < top returns with the i-th largest logit's expert in
// `id` and its softmax weight in `weight`.  NaN logits come out as experts in order with NaN weights.
template <int N>
__device__ __forceinline__ void choose_experts(const float *logits, uint32_t experts, uint32_t top, int lane, uint32_t *id, float *weight) {
    float v[N];
    bool bad = false;
    uint32_t taken = 0;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint32_t e = i * 64 + lane;
        v[i] = e < experts ? logits[e] : -INFINITY;
        if (e >= experts) taken |= 1u << i;
        bad = bad || v[i] != v[i];
        if (v[i] != v[i]) v[i] = -INFINITY;
    }
    bad = __any(bad);
    float mine = -INFINITY, first = 0.0f;
    *id = 0;
    for (uint32_t t = 0; t < top; ++t) {
        uint32_t at = 0;
        float value;
        take_largest<N>(v, taken, lane, &at, &value);
        if (t == 0) first = value;
        if ((uint32_t)lane == t) {
            mine = value;
            *id = at;
        }
    }
    const float e = (uint32_t)lane < top ? expf(mine - first) : 0.0f;
    const float sum = wave_sum_dpp(e);
    *weight = bad ? __uint_as_float(0x7fc00000u) : e / sum;
}

// The scored choice: softmax over all outputs, the `top` largest s + correction out of the best groups.  Lane i < top returns with
// the i-th chosen output in `id` and its weight in `weight`.  NaN: as above.
template <int N>
__device__ __forceinline__ void choose_scored(const float *logits, const RouteIo &io, int lane, uint32_t *id, float *weight) {
    float s[N], c[N], mx = -INFINITY, sum = 0.0f;
    bool bad = false;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint32_t e = i * 64 + lane;
        s[i] = e < io.experts ? logits[e] : -INFINITY;
        c[i] = e < io.experts ? io.correction[e] : 0.0f;
        bad = bad || s[i] != s[i];
        mx = fmaxf(mx, s[i]);
    }
    bad = __any(bad);
    mx = wave_max_dpp(mx);
#pragma unroll
    for (int i = 0; i < N; ++i) {
        s[i] = i * 64u + lane < io.experts ? expf(s[i] - mx) : 0.0f;
        sum += s[i];
    }
    sum = wave_sum_dpp(sum);
    uint32_t taken = 0;                              // bit i: this lane's value i cannot be chosen (any more)
#pragma unroll
    for (int i = 0; i < N; ++i) {
        s[i] /= sum;
        c[i] = bad ? 0.0f : s[i] + c[i];
        if (i * 64u + lane >= io.experts) taken |= 1u << i;
    }
    if (io.keep < io.groups) {
        // a group's best, then the number of groups ahead of it: value i of lane l belongs to group 64 i + l
        const uint32_t size = io.experts / io.groups;
        float best[N];
        uint32_t ahead[N];
#pragma unroll
        for (int i = 0; i < N; ++i) {
            best[i] = -INFINITY;
            ahead[i] = 0;
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            uint32_t g = i * 64 / size, left = size - i * 64 % size;
            const uint32_t n = io.experts > i * 64u ? (io.experts - i * 64 < 64 ? io.experts - i * 64 : 64) : 0;
            for (uint32_t l = 0; l < n; ++l) {
                const float v = lane_value(c[i], (int)l);
#pragma unroll
                for (int j = 0; j < N; ++j)
                    if (j * 64u + lane == g) best[j] = fmaxf(best[j], v);
                if (--left == 0) {
                    ++g;
                    left = size;
                }
            }
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const uint32_t n = io.groups > i * 64u ? (io.groups - i * 64 < 64 ? io.groups - i * 64 : 64) : 0;
            for (uint32_t l = 0; l < n; ++l) {
                const float v = lane_value(best[i], (int)l);
#pragma unroll
                for (int j = 0; j < N; ++j) ahead[j] += v > best[j] || (v == best[j] && i * 64u + l < j * 64u + lane);
            }
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const uint32_t g = (i * 64 + lane) / size;
            uint32_t rank = 0;
#pragma unroll
            for (int j = 0; j < N; ++j) {
                const uint32_t r = (uint32_t)__shfl((int)ahead[j], (int)(g % 64), 64);
                if (g / 64 == (uint32_t)j) rank = r;
            }
            if (rank >= io.keep) taken |= 1u << i;
        }
    }
    float mine = 0.0f;
    *id = 0;
    for (uint32_t t = 0; t < io.top; ++t) {
        uint32_t at = 0xffffffffu;
        float value, score = 0.0f;
        if (take_largest<N>(c, taken, lane, &at, &value)) {
#pragma unroll
            for (int i = 0; i < N; ++i)
                if (at / 64 == (uint32_t)i) score = lane_value(s[i], (int)(at % 64));
        }
        if ((uint32_t)lane == t) {
            mine = score;
            *id = at;
        }
    }
    const float total = wave_sum_dpp(mine) + 1e-20f;
    *weight = bad ? __uint_as_float(0x7fc00000u) : mine / total * io.scale;
}

// The experts of row r from its logits (LDS): gates stored; true in the lanes whose expert has a list.
// N: values per lane.
template <int N>
__device__ __forceinline__ bool choose_row(const float *logits, const RouteIo &io, uint64_t r, bool store, int lane, uint32_t *id) {
    float w;
    if (io.scored) choose_scored<N>(logits, io, lane, id, &w);
    else choose_experts<N>(logits, io.experts, io.top, lane, id, &w);
    const bool own = (uint32_t)lane < io.top, listed = own && *id < io.experts - io.identity;
    if (io.identity_gate) {
        const float sum = wave_sum_dpp(own && !listed ? w : 0.0f);
        if (store && lane == 0) io.identity_gate[r] = sum;
    }
    if (store && own) io.gate[r * io.top + lane] = listed ? w : 0.0f;
    return listed;
}

// ------------------------------------------------------------------ residual update
// One block per row, VPT pieces of it per thread: four values each (VEC, hidden a multiple of four), or one.
// KIND: ResidualNorm::Kind.
template <typename T, int VPT, int NT, bool ROUTE, bool VEC, int KIND>
__global__ void __launch_bounds__(NT)
    residual_norm_kernel(ResidualNorm rn, float *__restrict__ x, T *__restrict__ hn, uint32_t hidden, uint64_t ld, RouteIo io) {
    constexpr int NW = NT / 64, S = VEC ? 4 : 1;
    constexpr bool LAYER = KIND == ResidualNorm::kBoth, INPUT = KIND == ResidualNorm::kInput;
    typedef float piece __attribute__((ext_vector_type(S)));
    __shared__ float smem[LAYER ? 4 : 1][NW], logits[ROUTE ? kMaxExperts : 1];
    extern __shared__ __attribute__((aligned(16))) uint8_t hs_raw[];     // ROUTE: the row of hn
    const uint64_t r = blockIdx.x;
    const int tid = threadIdx.x;
    if (rn.clear && r == 0)
        for (uint32_t i = tid; i < rn.n_clear; i += NT) rn.clear[i] = 0;
    const float *y = rn.y + r * rn.parts * hidden;
    float *xr = x + r * hidden;
    piece v[VPT], xv[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const uint32_t c = (tid + i * NT) * S;
        v[i] = piece(0.0f);
        xv[i] = c < hidden ? *(const piece *)(xr + c) : piece(0.0f);
        if (!rn.gate && (!INPUT || rn.y) && c < hidden) v[i] = *(const piece *)(y + c);
    }
    if (rn.gate) {
        for (uint32_t p = 0; p < rn.parts; p += 2) {                     // two parts at a time, in order
            const bool two = p + 1 < rn.parts;
            const float g0 = rn.gate[r * rn.parts + p], g1 = two ? rn.gate[r * rn.parts + p + 1] : 0.0f;
            const float *y0 = y + (uint64_t)p * hidden, *y1 = two ? y0 + hidden : y0;
            piece t0[VPT], t1[VPT];
#pragma unroll
            for (int i = 0; i < VPT; ++i) {
                const uint32_t c = (tid + i * NT) * S;
                t0[i] = c < hidden && g0 != 0.0f ? *(const piece *)(y0 + c) : piece(0.0f);
                t1[i] = c < hidden && g1 != 0.0f ? *(const piece *)(y1 + c) : piece(0.0f);
            }
#pragma unroll
            for (int i = 0; i < VPT; ++i)
#pragma unroll
                for (int e = 0; e < S; ++e) v[i][e] = fmaf(g1, t1[i][e], fmaf(g0, t0[i][e], v[i][e]));
        }
        const float gi = rn.identity_gate ? rn.identity_gate[r] : 0.0f;
        if (gi != 0.0f) {
#pragma unroll
            for (int i = 0; i < VPT; ++i) {
                const uint32_t c = (tid + i * NT) * S;
                if (c >= hidden) continue;
                const T *h = hn + r * ld + c;
                piece t;
                if constexpr (sizeof(T) == 4) {
                    t = *(const piece *)h;
                } else if constexpr (VEC) {
                    const v2u b = *(const v2u *)h;
                    t = piece{bf16_lo(b[0]), bf16_hi(b[0]), bf16_lo(b[1]), bf16_hi(b[1])};
                } else {
                    t = piece(bf16_to_f32(*h));
                }
#pragma unroll
                for (int e = 0; e < S; ++e) v[i][e] = fmaf(gi, t[e], v[i][e]);
            }
        }
    }
    if constexpr (INPUT) {
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const uint32_t c = (tid + i * NT) * S;
            xv[i] += v[i];
            if (rn.y && c < hidden) *(piece *)(xr + c) = xv[i];
        }
        if (!rn.next) return;
    }
    // of the row behind v: its mean is taken off, the root of the mean square returned inverted
    auto center = [&](piece (&t)[VPT], float *s_mean, float *s_var) {
        if constexpr (LAYER) {
            float sum = 0.0f;
#pragma unroll
            for (int i = 0; i < VPT; ++i)
#pragma unroll
                for (int e = 0; e < S; ++e) sum += t[i][e];
            const float mean = block_sum<float, NW, true, true>(sum, s_mean) / (float)hidden;
#pragma unroll
            for (int i = 0; i < VPT; ++i)
                if ((uint32_t)(tid + i * NT) * S < hidden) t[i] -= mean;
        }
        float q = 0.0f;
#pragma unroll
        for (int i = 0; i < VPT; ++i)
#pragma unroll
            for (int e = 0; e < S; ++e) q = fmaf(t[i][e], t[i][e], q);
        return 1.0f / sqrtf(block_sum<float, NW, true, true>(q, s_var) / (float)hidden + rn.eps);
    };
    const float rstd = LAYER ? center(v, smem[LAYER], smem[0]) : center(INPUT ? xv : v, nullptr, smem[0]);
    if constexpr (LAYER) {
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const uint32_t c = (tid + i * NT) * S;
            if (c >= hidden) continue;
            const piece w = *(const piece *)(rn.w + c);
#pragma unroll
            for (int e = 0; e < S; ++e) xv[i][e] += v[i][e] * rstd * w[e];
            *(piece *)(xr + c) = xv[i];
        }
        if (!rn.next) return;
        const float r2 = center(xv, smem[LAYER ? 2 : 0], smem[LAYER ? 3 : 0]);
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const uint32_t c = (tid + i * NT) * S;
            if (c >= ld) continue;
            piece o = piece(0.0f);
            if (c < hidden) o = xv[i] * r2 * *(const piece *)(rn.next + c);
            T *dst = hn + r * ld + c;
            if constexpr (sizeof(T) == 4) *(piece *)dst = o;
            else if constexpr (VEC) *(v2u *)dst = v2u{f32x2_to_bf16x2(o[0], o[1]), f32x2_to_bf16x2(o[2], o[3])};
            else *dst = f32_to_bf16(o[0]);
        }
        return;
    }
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const uint32_t c = (tid + i * NT) * S;
        if (c >= ld) continue;
        piece o = piece(0.0f);
        if (INPUT) {
            if (c < hidden) o = xv[i] * rstd * *(const piece *)(rn.next + c);
        } else if (c < hidden) {
            const piece w = *(const piece *)(rn.w + c);
#pragma unroll
            for (int e = 0; e < S; ++e) o[e] = xv[i][e] + v[i][e] * rstd * w[e];
            *(piece *)(xr + c) = o;
        }
        auto put = [&](T *dst) {
            if constexpr (sizeof(T) == 4) *(piece *)dst = o;
            else if constexpr (VEC) *(v2u *)dst = v2u{f32x2_to_bf16x2(o[0], o[1]), f32x2_to_bf16x2(o[2], o[3])};
            else *dst = f32_to_bf16(o[0]);
        };
        put(hn + r * ld + c);
        if constexpr (ROUTE) put((T *)hs_raw + c);
    }
    if constexpr (ROUTE) {
        const int lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64);
        const T *h = (const T *)hs_raw;
        __syncthreads();
        if constexpr (sizeof(T) == 4) {
            for (uint32_t e = wave; e < io.experts; e += NW) {
                const float *w = (const float *)io.w + (uint64_t)e * ld;
                float acc = 0.0f;
                for (uint32_t c = lane; c < ld; c += 64) acc = fmaf(w[c], h[c], acc);
                const float z = wave_sum_dpp(acc);
                if (lane == 0) logits[e] = z;
            }
        } else {
            // every wavefront its k tiles of all experts; the row is the operand of all sixteen columns
            float *part = (float *)(hs_raw + ld * sizeof(T));        // [experts padded to 16][NW + 1]
            const uint32_t k_tiles = (uint32_t)(ld / 32), tiles = (io.experts + 15) / 16;
            for (uint32_t t = 0; t < tiles; ++t) {
                const v8bf *w = (const v8bf *)io.w + (uint64_t)t * k_tiles * 64 + lane;
                v4f acc = v4f{0.f, 0.f, 0.f, 0.f};
                for (uint32_t s0 = wave; s0 < k_tiles; s0 += NW * 4) {
                    v8bf wv[4];
#pragma unroll
                    for (int u = 0; u < 4; ++u) wv[u] = w[(uint64_t)(s0 + u * NW < k_tiles ? s0 + u * NW : s0) * 64];
#pragma unroll
                    for (int u = 0; u < 4; ++u) {
                        const uint32_t s = s0 + u * NW;
                        if (s < k_tiles) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u], *(const v8bf *)(h + s * 32 + 8 * (lane / 16)), acc, 0, 0, 0);
                    }
                }
                if (lane % 16 == 0)
#pragma unroll
                    for (int e = 0; e < 4; ++e) part[(t * 16 + 4 * (lane / 16) + e) * (NW + 1) + wave] = acc[e];
            }
            __syncthreads();
            for (uint32_t e = tid; e < io.experts; e += NT) {
                float z = 0.0f;
#pragma unroll
                for (int q = 0; q < NW; ++q) z += part[e * (NW + 1) + q];
                logits[e] = z;
            }
        }
        __syncthreads();
        if (wave == 0) {
            uint32_t id;
            if (io.experts <= 64 ? choose_row<1>(logits, io, r, true, lane, &id) : choose_row<kMaxExperts / 64>(logits, io, r, true, lane, &id)) {
                const uint32_t at = atomicAdd(io.count + id, 1u);
                if (at < io.pitch) io.list[(uint64_t)id * io.pitch + at] = (uint32_t)(r * io.top + lane);
            }
        }
    }
}

// ------------------------------------------------------------------ router
// 16 rows per block; its four wavefronts take a quarter of k each and meet in LDS.  ET: tiles of 16 experts, those past the
// weight's last one repeat it (nobody looks at their logits).
template <int ET>
__global__ void __launch_bounds__(256)
    route_kernel(const uint16_t *__restrict__ h, uint64_t ld, uint32_t rows, RouteIo io) {
    extern __shared__ __attribute__((aligned(16))) float part[];         // [4][ET * 16][17]
    __shared__ uint32_t cnt[kMaxExperts], base[kMaxExperts];
    __shared__ float logits[16][ET * 16 + 1];
    const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), g = lane / 16, c = lane % 16;
    const uint32_t r0 = blockIdx.x * 16, row = r0 + c < rows ? r0 + c : rows - 1;
    const uint16_t *hp = h + (uint64_t)row * ld + 8 * g, *wp = (const uint16_t *)io.w + lane * 8;
    v4f acc[ET];
#pragma unroll
    for (int t = 0; t < ET; ++t) acc[t] = v4f{0.f, 0.f, 0.f, 0.f};
    const uint32_t steps = (uint32_t)(ld / 32), last_tile = (io.experts + 15) / 16 - 1;
    constexpr int U = ET == 1 ? 8 : ET == 2 ? 4 : ET == 4 ? 2 : 1;       // k steps whose loads are in flight together
    for (uint32_t s0 = wave; s0 < steps; s0 += 4 * U) {
        v8bf hv[U], wv[U][ET];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const uint32_t s = s0 + 4 * u < steps ? s0 + 4 * u : s0;
            hv[u] = *(const v8bf *)(hp + (uint64_t)s * 32);
#pragma unroll
            for (int t = 0; t < ET; ++t) wv[u][t] = *(const v8bf *)(wp + ((uint64_t)((uint32_t)t < last_tile ? t : last_tile) * steps + s) * 512);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (s0 + 4 * u < steps) {
#pragma unroll
                for (int t = 0; t < ET; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u][t], hv[u], acc[t], 0, 0, 0);
            }
    }
#pragma unroll
    for (int t = 0; t < ET; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) part[(wave * ET * 16 + t * 16 + 4 * g + e) * 17 + c] = acc[t][e];
    for (uint32_t i = tid; i < kMaxExperts; i += 256) cnt[i] = 0;
    __syncthreads();
    for (int i = tid; i < ET * 256; i += 256) {
        const int e = i / 16, rr = i % 16;
        logits[rr][e] = (part[e * 17 + rr] + part[(ET * 16 + e) * 17 + rr]) + (part[(2 * ET * 16 + e) * 17 + rr] + part[(3 * ET * 16 + e) * 17 + rr]);
    }
    __syncthreads();
    uint32_t id[4], at[4];
    bool listed[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        const uint32_t rr = wave * 4 + q;
        const bool there = r0 + rr < rows;
        listed[q] = choose_row<(ET + 3) / 4>(logits[rr], io, r0 + rr, there, lane, &id[q]) && there;
        at[q] = listed[q] ? atomicAdd(&cnt[id[q]], 1u) : 0;
    }
    __syncthreads();
    for (uint32_t e = tid; e < io.experts - io.identity; e += 256)
        if (cnt[e]) base[e] = atomicAdd(io.count + e, cnt[e]);
    __syncthreads();
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        const uint32_t rr = wave * 4 + q;
        if (listed[q]) {
            const uint32_t p = base[id[q]] + at[q];
            if (p < io.pitch) io.list[(uint64_t)id[q] * io.pitch + p] = (uint32_t)((r0 + rr) * io.top + lane);
        }
    }
}

template <typename T, int VPT, int NT, bool ROUTE, bool VEC, int KIND>
void launch_residual_kind(const ResidualNorm &rn, float *x, T *hn, uint64_t rows, uint64_t hidden, uint64_t ld, const RouteIo &io, hipStream_t s) {
    const size_t lds = ROUTE ? ld * sizeof(T) + (sizeof(T) == 2 ? (io.experts + 15) / 16 * 16 * 17 * 4 : 0) : 0;
    if (ROUTE && lds > 49152) {
        static bool configured = false;
        if (!configured) {
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&residual_norm_kernel<T, VPT, NT, ROUTE, VEC, KIND>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                      98304);
            configured = true;
        }
    }
    residual_norm_kernel<T, VPT, NT, ROUTE, VEC, KIND><<<(unsigned)rows, NT, lds, s>>>(rn, x, hn, (uint32_t)hidden, ld, io);
}
template <typename T, int VPT, int NT, bool ROUTE, bool VEC>
void launch_residual_sized(const ResidualNorm &rn, float *x, T *hn, uint64_t rows, uint64_t hidden, uint64_t ld, const RouteIo &io, hipStream_t s) {
    if constexpr (!ROUTE)
        if (rn.kind == ResidualNorm::kBoth) return launch_residual_kind<T, VPT, NT, false, VEC, ResidualNorm::kBoth>(rn, x, hn, rows, hidden, ld, io, s);
    if (rn.kind == ResidualNorm::kInput) launch_residual_kind<T, VPT, NT, ROUTE, VEC, ResidualNorm::kInput>(rn, x, hn, rows, hidden, ld, io, s);
    else launch_residual_kind<T, VPT, NT, ROUTE, VEC, ResidualNorm::kOutput>(rn, x, hn, rows, hidden, ld, io, s);
}

// rows up to 16384 values
template <typename T, bool ROUTE>
void launch_residual(const ResidualNorm &rn, float *x, T *hn, uint64_t rows, uint64_t hidden, uint64_t ld, const RouteIo &io, hipStream_t s) {
    if (hidden % 4 == 0) {
        if (ld <= 1024) launch_residual_sized<T, 1, 256, ROUTE, true>(rn, x, hn, rows, hidden, ld, io, s);
        else if (rows > 256 && ld <= 4096) launch_residual_sized<T, 4, 256, ROUTE, true>(rn, x, hn, rows, hidden, ld, io, s);
        else if (ld <= 4096) launch_residual_sized<T, 1, 1024, ROUTE, true>(rn, x, hn, rows, hidden, ld, io, s);
        else launch_residual_sized<T, 4, 1024, ROUTE, true>(rn, x, hn, rows, hidden, ld, io, s);
    } else {
        if (ld <= 1024) launch_residual_sized<T, 4, 256, ROUTE, false>(rn, x, hn, rows, hidden, ld, io, s);
        else launch_residual_sized<T, 16, 1024, ROUTE, false>(rn, x, hn, rows, hidden, ld, io, s);
    }
}

template <int ET>
void launch_route(const uint16_t *h, uint64_t rows, uint64_t ld, const RouteIo &io, hipStream_t s) {
    constexpr int lds = 4 * ET * 16 * 17 * 4;
    if constexpr (lds + ET * 1024 > 49152) {
        static bool configured = false;
        if (!configured) {
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&route_kernel<ET>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
            configured = true;
        }
    }
    route_kernel<ET><<<(unsigned)((rows + 15) / 16), 256, lds, s>>>(h, ld, (uint32_t)rows, io);
}

}  // namespace

bool residual_norm_routes(int is_f32, uint64_t rows) { return is_f32 || g_route_form == 1 || (rows <= 64 && g_route_form != 2); }

void residual_norm(const ResidualNorm &rn, float *x, void *hn, int is_f32, uint64_t rows, uint64_t hidden, uint64_t ld, const RouteIo *route,
                   hipStream_t s) {
    if (rows == 0) return;
    if (is_f32) {
        if (route) launch_residual<float, true>(rn, x, (float *)hn, rows, hidden, ld, *route, s);
        else launch_residual<float, false>(rn, x, (float *)hn, rows, hidden, ld, RouteIo{}, s);
    } else {
        if (route) launch_residual<uint16_t, true>(rn, x, (uint16_t *)hn, rows, hidden, ld, *route, s);
        else launch_residual<uint16_t, false>(rn, x, (uint16_t *)hn, rows, hidden, ld, RouteIo{}, s);
    }
}

namespace {
__global__ void xielu_constants_kernel(const float *pq, float *act) {
    const float z = pq[threadIdx.x];
    act[threadIdx.x] = fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))) + (threadIdx.x ? 0.5f : 0.0f);
}
}  // namespace
void xielu_constants(const float *pq, float *act, hipStream_t s) { xielu_constants_kernel<<<1, 2, 0, s>>>(pq, act); }

void route_rows(const void *h_bf16, uint64_t rows, uint64_t ld, const RouteIo &io, hipStream_t s) {
    if (rows == 0) return;
    const uint16_t *p = (const uint16_t *)h_bf16;
    if (io.experts <= 16) launch_route<1>(p, rows, ld, io, s);
    else if (io.experts <= 32) launch_route<2>(p, rows, ld, io, s);
    else if (io.experts <= 64) launch_route<4>(p, rows, ld, io, s);
    else if (io.experts <= 128) launch_route<8>(p, rows, ld, io, s);
    else launch_route<16>(p, rows, ld, io, s);
}

}  // namespace k
}  // namespace fa
