// Mixture of experts: a narrow product with 32-bit results (router logits), the choice of experts, the list of every
// expert's tokens, and the experts' products over those lists.
//
// An item is (token, place among its chosen experts), numbered token * top + place.  Products write their row of an item
// at the item's number, so nothing is sorted in memory: the lists say which rows an expert reads and writes, and the
// weighted sum over a token's items happens where the result is used (pa_residual_norm).  No counts go through the host.
//
// Product kernels, by how many tokens an expert has on average: tiles through LDS (the loads go straight to LDS, two
// buffers, one barrier per 64 elements of the inner dimension), or, for a few tokens per expert, weights streamed from
// memory into registers.  The weights' rows are zero-padded to whole 64-element steps; token rows are not read past
// their end.  All products are taken transposed (weight rows as the rows of the result), so that a lane holds four
// consecutive outputs of one item.
#include "moe_plan.h"
#include "row_common.h"

namespace {

typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef float f4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f4 moe_mfma(bf8 x, bf8 y, f4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, y, c, 0, 0, 0); }
__device__ __forceinline__ bf8 moe_load(const uint16_t *p) { return *reinterpret_cast<const bf8 *>(p); }
__device__ __forceinline__ bf8 moe_zero() { return __builtin_bit_cast(bf8, make_uint4(0, 0, 0, 0)); }

// ------------------------------------------------------------------ narrow product, 32-bit results
struct NarrowArgs {
    const void *x, *w;  // [rows][ldx], [n][k]
    int64_t ldx;
    float *out;  // [rows][n]
    int64_t rows;
    int n, k;
};

// 16 RT rows x 64 columns per workgroup; its NW waves share the inner dimension.  (k: whole 16-byte vectors)
template <int RT, int NW> __global__ __launch_bounds__(64 * NW) void narrow_mfma_kernel(const NarrowArgs a) {
    __shared__ float red[NW / 2][RT * 16][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    const int64_t r0 = (int64_t)blockIdx.x * 16 * RT;
    const int n0 = blockIdx.y * 64;
    const uint16_t *xr[RT], *wr[4];
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const int64_t r = r0 + 16 * t + l16;
        xr[t] = reinterpret_cast<const uint16_t *>(a.x) + (r < a.rows ? r : a.rows - 1) * a.ldx;
    }
#pragma unroll
    for (int c = 0; c < 4; ++c) {
        const int n = n0 + 16 * c + l16;
        wr[c] = reinterpret_cast<const uint16_t *>(a.w) + (int64_t)(n < a.n ? n : a.n - 1) * a.k;
    }
    f4 acc[RT][4];
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[t][c] = f4{0.f, 0.f, 0.f, 0.f};
    // (the four lanes of a row take 32 consecutive bytes each: whole lines, in the same order for both operands)
    for (int k0 = 64 * wave; k0 < a.k; k0 += 64 * NW) {
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int k = k0 + 16 * g + 8 * half;
            const bool in = k < a.k;
            bf8 x[RT];
#pragma unroll
            for (int t = 0; t < RT; ++t) x[t] = in ? moe_load(xr[t] + k) : moe_zero();
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                const bf8 w = in ? moe_load(wr[c] + k) : moe_zero();
#pragma unroll
                for (int t = 0; t < RT; ++t) acc[t][c] = moe_mfma(w, x[t], acc[t][c]);
            }
        }
    }
#pragma unroll
    for (int step = NW / 2; step >= 1; step /= 2) {
        if (wave >= step && wave < 2 * step) {
#pragma unroll
            for (int t = 0; t < RT; ++t)
#pragma unroll
                for (int c = 0; c < 4; ++c)
#pragma unroll
                    for (int i = 0; i < 4; ++i) red[wave - step][(t * 4 + c) * 4 + i][lane] = acc[t][c][i];
        }
        __syncthreads();
        if (wave < step) {
#pragma unroll
            for (int t = 0; t < RT; ++t)
#pragma unroll
                for (int c = 0; c < 4; ++c)
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc[t][c][i] += red[wave][(t * 4 + c) * 4 + i][lane];
        }
        __syncthreads();
    }
    if (wave != 0) return;
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const int64_t r = r0 + 16 * t + l16;
        if (r >= a.rows) continue;
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = n0 + 16 * c + 4 * g + i;
                if (n < a.n) a.out[r * a.n + n] = acc[t][c][i];
            }
    }
}

// One wave per result
template <typename T> __global__ __launch_bounds__(256) void narrow_dot_kernel(const NarrowArgs a) {
    const int64_t r = blockIdx.x;
    const int n = blockIdx.y * 4 + threadIdx.x / 64, lane = threadIdx.x & 63;
    if (n >= a.n) return;
    const T *x = reinterpret_cast<const T *>(a.x) + r * a.ldx, *w = reinterpret_cast<const T *>(a.w) + (int64_t)n * a.k;
    float acc = 0.f;
    for (int k = lane; k < a.k; k += 64) acc = fmaf(pa_scalar<T>::load(x + k), pa_scalar<T>::load(w + k), acc);
    acc = pa_group_sum<64>(acc);
    if (lane == 0) a.out[r * a.n + n] = acc;
}

// ------------------------------------------------------------------ choice of experts
struct SelectArgs {
    const float *logits;  // [rows][ld]: the experts', then (shared) one for the shared expert's gate
    int64_t ld, rows;
    int32_t *ids;    // [rows][top]
    float *weights;  // [rows][top + 1], the last one the shared expert's
    int experts, top, groups, keep, shared;
};

// Position of the largest of `n` values in LDS, the lowest on ties, or n when all are NaN; every lane of the wave gets it.
__device__ __forceinline__ int moe_argmax(const float *v, int n, int lane) {
    float best = -3.f;
    int at = n;
    for (int i = lane; i < n; i += 64)
        if (v[i] > best) {
            best = v[i];
            at = i;
        }
#pragma unroll
    for (int d = 32; d >= 1; d /= 2) {
        const float ob = __shfl_xor(best, d, 64);
        const int oa = __shfl_xor(at, d, 64);
        if (ob > best || (ob == best && oa < at)) {
            best = ob;
            at = oa;
        }
    }
    return at;
}

// One wave per row, four rows per workgroup (all of them run the same number of barriers).
__global__ __launch_bounds__(256) void moe_select_kernel(const SelectArgs a) {
    extern __shared__ float sel[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x / 64;
    float *score = sel + wave * (a.experts + a.groups), *value = score + a.experts;
    const int64_t row = (int64_t)blockIdx.x * 4 + wave;
    const bool live = row < a.rows;
    const float *logit = a.logits + (live ? row : 0) * a.ld;
    for (int e = lane; e < a.experts; e += 64) score[e] = 1.f / (1.f + expf(-logit[e]));
    __syncthreads();
    if (a.keep < a.groups) {
        const int size = a.experts / a.groups;
        for (int g = lane; g < a.groups; g += 64) {  // a group's value: its two largest scores
            float one = 0.f, two = 0.f;
            for (int e = g * size; e < (g + 1) * size; ++e) {
                const float s = score[e];
                if (s > one) {
                    two = one;
                    one = s;
                } else {
                    two = fmaxf(two, s);
                }
            }
            value[g] = one + two;
        }
        __syncthreads();
        for (int i = 0; i < a.keep; ++i) {  // kept groups: value -1
            const int at = moe_argmax(value, a.groups, lane);
            __syncthreads();
            if (lane == 0 && at < a.groups) value[at] = -1.f;
            __syncthreads();
        }
        for (int e = lane; e < a.experts; e += 64)
            if (value[e / size] >= 0.f) score[e] = -1.f;
        __syncthreads();
    }
    float sum = 0.f, mine = 0.f;
    for (int i = 0; i < a.top; ++i) {
        const int at = moe_argmax(score, a.experts, lane);
        const bool found = at < a.experts;  // (a row of NaN has no experts)
        const float s = found ? score[at] : 0.f;
        sum += s;
        if (lane == i) mine = s;
        __syncthreads();
        if (lane == 0) {
            if (found) score[at] = -2.f;
            if (live) a.ids[row * a.top + i] = found && s >= 0.f ? at : -1;
        }
        __syncthreads();
    }
    if (!live) return;
    if (lane < a.top) a.weights[row * (a.top + 1) + lane] = mine / (sum + 1e-20f);
    if (lane == 0) a.weights[row * (a.top + 1) + a.top] = a.shared ? 1.f / (1.f + expf(-logit[a.experts])) : 0.f;
}

// ------------------------------------------------------------------ lists
constexpr int kListThreads = 1024, kListPer = 16;

// Workgroup e lists the items of expert e in their order: lists[e][0 .. counts[e])
__global__ __launch_bounds__(kListThreads) void moe_lists_kernel(const int32_t *ids, int64_t items, int64_t cap, int32_t *counts, int32_t *lists) {
    __shared__ int waves[kListThreads / 64];
    const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid / 64;
    int32_t *out = lists + e * cap;
    int base = 0;
    for (int64_t at = 0; at < items; at += (int64_t)kListThreads * kListPer) {
        const int64_t first = at + (int64_t)tid * kListPer;
        uint32_t hit = 0;
#pragma unroll
        for (int i = 0; i < kListPer; i += 4) {
            int4 v = make_int4(-1, -1, -1, -1);
            if (first + i + 3 < items) {
                v = *reinterpret_cast<const int4 *>(ids + first + i);
            } else {
                if (first + i < items) v.x = ids[first + i];
                if (first + i + 1 < items) v.y = ids[first + i + 1];
                if (first + i + 2 < items) v.z = ids[first + i + 2];
            }
            hit |= (uint32_t)(v.x == e) << i | (uint32_t)(v.y == e) << (i + 1) | (uint32_t)(v.z == e) << (i + 2) |
                   (uint32_t)(v.w == e) << (i + 3);
        }
        const int n = __popc(hit);
        int upto = n;
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const int y = __shfl_up(upto, d, 64);
            if (lane >= d) upto += y;
        }
        if (lane == 63) waves[wave] = upto;
        __syncthreads();
        int before = base, total = 0;
#pragma unroll
        for (int w = 0; w < kListThreads / 64; ++w) {
            if (w < wave) before += waves[w];
            total += waves[w];
        }
        int64_t to = before + upto - n;
        for (; hit; hit &= hit - 1, ++to)
            if (to < cap) out[to] = (int32_t)(first + __ffs(hit) - 1);
        base += total;
        __syncthreads();
    }
    if (tid == 0) counts[e] = base < cap ? base : (int)cap;
}

// ------------------------------------------------------------------ products
struct MoeArgs {
    const void *x;  // item i reads row i / per_row at row stride ldx
    int64_t ldx;
    int per_row;
    const void *w;  // [experts][w_rows][kp]
    int64_t w_rows;
    int k, kp, n;   // elements of a row of x, of a row of w (zeros past k), outputs per item
    const int32_t *counts, *lists;
    int64_t cap, items;
    int experts;
    void *out;  // [items][n]
};

// The `tile`-th tile of `bm` items over all experts: expert and first place in its list; false when there are fewer.
// Every wave finds it by itself.
__device__ __forceinline__ bool moe_tile(const MoeArgs &a, int tile, int bm, int lane, int &expert, int &m0, int &count) {
    int before = 0;
    for (int e0 = 0; e0 < a.experts; e0 += 64) {
        const int e = e0 + lane, c = e < a.experts ? a.counts[e] : 0, t = (c + bm - 1) / bm;
        int upto = t;
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const int y = __shfl_up(upto, d, 64);
            if (lane >= d) upto += y;
        }
        const uint64_t past = __ballot(before + upto > tile);
        if (past) {
            const int l = __ffsll((unsigned long long)past) - 1;
            expert = __builtin_amdgcn_readfirstlane(e0 + l);
            count = __builtin_amdgcn_readfirstlane(__shfl(c, l, 64));
            m0 = __builtin_amdgcn_readfirstlane((tile - before - __shfl(upto - t, l, 64)) * bm);
            return true;
        }
        before += __shfl(upto, 63, 64);
    }
    return false;
}

__device__ __forceinline__ uint32_t moe_glu2(float g0, float u0, float g1, float u1) {
    return row_pack_bf16(row_silu<pa_bf16>(g0) * u0, row_silu<pa_bf16>(g1) * u1);
}

// Consecutive workgroups go to the dies in turn; this gives a die consecutive tiles, which share weights and items.
__device__ __forceinline__ int moe_swizzle(int i, int total) {
    const int per = total / 8;
    return i < per * 8 ? i % 8 * per + i / 8 : i;
}

typedef __attribute__((address_space(3))) void *lds_ptr;
typedef const __attribute__((address_space(1))) void *global_ptr;

// WM x WN waves; a wave holds TM tiles of 16 items by TN tiles of 16 weight rows.  GLU: the workgroup's weight rows are half
// gate, half up rows of the same outputs, and a wave's tiles likewise.
template <int TM, int TN, int WM, int WN, bool GLU>
__global__ __launch_bounds__(64 * WM * WN, 2) void moe_tile_kernel(const MoeArgs a) {
    constexpr int kBM = 16 * TM * WM, kBN = 16 * TN * WN, kWaves = WM * WN, kThr = 64 * kWaves;
    constexpr int kLoadsA = kBM / 8 / kWaves, kLoadsB = kBN / 8 / kWaves;  // wave-wide loads of eight 128-byte rows
    static_assert(kBM % (8 * kWaves) == 0 && kBN % (8 * kWaves) == 0 && (!GLU || TN % 2 == 0), "whole loads per wave");
    extern __shared__ __align__(16) char lds[];
    __bf16 *as = reinterpret_cast<__bf16 *>(lds), *bs = as + 2 * kBM * 64;  // rows of eight 16-byte chunks, chunk c of row r at c ^ (r & 7)
    int32_t *item_s = reinterpret_cast<int32_t *>(bs + 2 * kBN * 64);
    constexpr int kOut = GLU ? kBN / 2 : kBN;  // outputs per workgroup
    const int n_tiles = (a.n + kOut - 1) / kOut;
    const int i = moe_swizzle(blockIdx.x, gridDim.x);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    int expert, m0, count;
    if (!moe_tile(a, i / n_tiles, kBM, lane, expert, m0, count)) return;
    const int n0 = i % n_tiles * kOut;
    for (int j = tid; j < kBM; j += kThr) {
        const int32_t item = m0 + j < count ? a.lists[expert * a.cap + m0 + j] : -1;
        item_s[j] = item >= 0 && item < a.items ? item : -1;
    }
    __syncthreads();
    // sources of this lane's chunks
    const int r8 = lane / 8, ch = (lane % 8) ^ r8;
    const uint16_t *x = reinterpret_cast<const uint16_t *>(a.x), *w = reinterpret_cast<const uint16_t *>(a.w) + expert * a.w_rows * a.kp;
    const uint16_t *pa[kLoadsA], *pb[kLoadsB];
#pragma unroll
    for (int j = 0; j < kLoadsA; ++j) {
        const int item = item_s[(wave * kLoadsA + j) * 8 + r8];
        pa[j] = x + (int64_t)((item < 0 ? 0 : item) / a.per_row) * a.ldx;
    }
#pragma unroll
    for (int j = 0; j < kLoadsB; ++j) {
        const int r = (wave * kLoadsB + j) * 8 + r8;
        int n = n0 + (GLU ? r % (kBN / 2) : r);
        if (n >= a.n) n = a.n - 1;
        if (GLU && r >= kBN / 2) n += a.n;
        pb[j] = w + (int64_t)n * a.kp + 8 * ch;
    }
    auto fetch = [&](int k0, int buf) {
        const int k = k0 + 8 * ch;
#pragma unroll
        for (int j = 0; j < kLoadsA; ++j)  // (past a row's end: its first elements, against zeros of the weights)
            __builtin_amdgcn_global_load_lds((global_ptr)(pa[j] + (k < a.k ? k : 0)),
                                             (lds_ptr)(as + (buf * kBM + (wave * kLoadsA + j) * 8) * 64), 16, 0, 0);
#pragma unroll
        for (int j = 0; j < kLoadsB; ++j)
            __builtin_amdgcn_global_load_lds((global_ptr)(pb[j] + k0),
                                             (lds_ptr)(bs + (buf * kBN + (wave * kLoadsB + j) * 8) * 64), 16, 0, 0);
    };
    const int wm = wave / WN, wn = wave % WN;
    f4 acc[TN][TM];
#pragma unroll
    for (int t = 0; t < TN; ++t)
#pragma unroll
        for (int m = 0; m < TM; ++m) acc[t][m] = f4{0.f, 0.f, 0.f, 0.f};
    // first weight row of the wave's tile t
    auto tile_row = [&](int t) { return GLU ? (t < TN / 2 ? 16 * (wn * TN / 2 + t) : kBN / 2 + 16 * (wn * TN / 2 + t - TN / 2)) : 16 * (wn * TN + t); };
    fetch(0, 0);
    for (int k0 = 0, buf = 0; k0 < a.kp; k0 += 64, buf ^= 1) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();  // this step's tiles are there; the other buffer has been read
        if (k0 + 64 < a.kp) fetch(k0 + 64, buf ^ 1);
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const int c8 = ((kk * 4 + g) ^ (l16 & 7)) * 8;
            bf8 xa[TM];
#pragma unroll
            for (int m = 0; m < TM; ++m)
                xa[m] = *reinterpret_cast<const bf8 *>(as + (buf * kBM + 16 * (wm * TM + m) + l16) * 64 + c8);
#pragma unroll
            for (int t = 0; t < TN; ++t) {
                const bf8 wb = *reinterpret_cast<const bf8 *>(bs + (buf * kBN + tile_row(t) + l16) * 64 + c8);
#pragma unroll
                for (int m = 0; m < TM; ++m) acc[t][m] = moe_mfma(wb, xa[m], acc[t][m]);
            }
        }
    }
    uint16_t *out = reinterpret_cast<uint16_t *>(a.out);
#pragma unroll
    for (int m = 0; m < TM; ++m) {
        const int item = item_s[16 * (wm * TM + m) + l16];
        if (item < 0) continue;
        uint16_t *row = out + (int64_t)item * a.n;
#pragma unroll
        for (int t = 0; t < (GLU ? TN / 2 : TN); ++t) {
            const int n = n0 + 16 * ((GLU ? wn * TN / 2 : wn * TN) + t) + 4 * g;
            if (n >= a.n) continue;  // (n: whole groups of four)
            const f4 y = acc[t][m];
            uint2 p;
            if constexpr (GLU) {
                const f4 u = acc[t + TN / 2][m];
                p = make_uint2(moe_glu2(y[0], u[0], y[1], u[1]), moe_glu2(y[2], u[2], y[3], u[3]));
            } else {
                p = make_uint2(row_pack_bf16(y[0], y[1]), row_pack_bf16(y[2], y[3]));
            }
            *reinterpret_cast<uint2 *>(row + n) = p;
        }
    }
}

// A few items per expert: every wave streams two tiles of 16 weight rows (GLU: the gate and up rows of the same outputs)
// past MT tiles of 16 items.
template <int MT, bool GLU> __global__ __launch_bounds__(256) void moe_stream_kernel(const MoeArgs a) {
    constexpr int kOut = GLU ? 64 : 128;  // outputs per workgroup
    const int n_tiles = (a.n + kOut - 1) / kOut;
    const int i = moe_swizzle(blockIdx.x, gridDim.x);
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    int expert, m0, count;
    if (!moe_tile(a, i / n_tiles, 16 * MT, lane, expert, m0, count)) return;
    const int n0 = i % n_tiles * kOut + wave * (GLU ? 16 : 32);
    if (n0 >= a.n) return;
    const uint16_t *w = reinterpret_cast<const uint16_t *>(a.w) + expert * a.w_rows * a.kp + 16 * g;
    auto w_row = [&](int n) { return w + (int64_t)(n < a.n ? n : a.n - 1) * a.kp; };
    const uint16_t *w0 = w_row(n0 + l16), *w1 = GLU ? w0 + (int64_t)a.n * a.kp : w_row(n0 + 16 + l16);
    const uint16_t *x[MT];
    int items[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int place = m0 + 16 * m + l16;
        const int32_t item = place < count ? a.lists[expert * a.cap + place] : -1;
        items[m] = item >= 0 && item < a.items ? item : -1;
        x[m] = reinterpret_cast<const uint16_t *>(a.x) + (int64_t)((items[m] < 0 ? 0 : items[m]) / a.per_row) * a.ldx;
    }
    f4 acc[2][MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[0][m] = acc[1][m] = f4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.kp; k0 += 64) {
        // (the four lanes of a row take 32 consecutive bytes each: whole lines, in the same order for both operands)
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int k = k0 + 16 * g + 8 * half;
            const bf8 b0 = moe_load(w0 + k0 + 8 * half), b1 = moe_load(w1 + k0 + 8 * half);
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                const bf8 y = moe_load(x[m] + (k < a.k ? k : 0));
                acc[0][m] = moe_mfma(b0, y, acc[0][m]);
                acc[1][m] = moe_mfma(b1, y, acc[1][m]);
            }
        }
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        if (items[m] < 0) continue;
        uint16_t *row = reinterpret_cast<uint16_t *>(a.out) + (int64_t)items[m] * a.n;
        const f4 y = acc[0][m], z = acc[1][m];
        const int n = n0 + 4 * g;
        if constexpr (GLU) {
            if (n < a.n)
                *reinterpret_cast<uint2 *>(row + n) = make_uint2(moe_glu2(y[0], z[0], y[1], z[1]), moe_glu2(y[2], z[2], y[3], z[3]));
        } else {
            if (n < a.n) *reinterpret_cast<uint2 *>(row + n) = make_uint2(row_pack_bf16(y[0], y[1]), row_pack_bf16(y[2], y[3]));
            if (n + 16 < a.n)
                *reinterpret_cast<uint2 *>(row + n + 16) = make_uint2(row_pack_bf16(z[0], z[1]), row_pack_bf16(z[2], z[3]));
        }
    }
}

// 32-bit rows, and rows that are not whole vectors: 16 items x 64 outputs per workgroup, four items per thread.
template <typename T, bool GLU> __global__ __launch_bounds__(256) void moe_vector_kernel(const MoeArgs a) {
    constexpr int kStep = 32;
    __shared__ float xs[16][kStep + 1], ws[GLU ? 2 : 1][64][kStep + 1];
    __shared__ int32_t item_s[16];
    const int n_tiles = (a.n + 63) / 64;
    const int tid = threadIdx.x, col = tid % 64, grp = tid / 64;
    int expert, m0, count;
    if (!moe_tile(a, blockIdx.x / n_tiles, 16, tid & 63, expert, m0, count)) return;
    const int n0 = blockIdx.x % n_tiles * 64;
    if (tid < 16) {
        const int32_t item = m0 + tid < count ? a.lists[expert * a.cap + m0 + tid] : -1;
        item_s[tid] = item >= 0 && item < a.items ? item : -1;
    }
    __syncthreads();
    const T *x = reinterpret_cast<const T *>(a.x), *w = reinterpret_cast<const T *>(a.w) + expert * a.w_rows * a.kp;
    float acc[GLU ? 2 : 1][4] = {};
    for (int k0 = 0; k0 < a.k; k0 += kStep) {
        for (int j = tid; j < 16 * kStep; j += 256) {
            const int r = j / kStep, k = k0 + j % kStep, item = item_s[r];
            xs[r][j % kStep] = item >= 0 && k < a.k ? pa_scalar<T>::load(x + (int64_t)(item / a.per_row) * a.ldx + k) : 0.f;
        }
        for (int j = tid; j < 64 * kStep; j += 256) {
            const int r = j / kStep, k = k0 + j % kStep, n = n0 + r;
            const bool in = n < a.n && k < a.k;
            ws[0][r][j % kStep] = in ? pa_scalar<T>::load(w + (int64_t)n * a.kp + k) : 0.f;
            if constexpr (GLU) ws[1][r][j % kStep] = in ? pa_scalar<T>::load(w + (int64_t)(a.n + n) * a.kp + k) : 0.f;
        }
        __syncthreads();
        for (int k = 0; k < kStep; ++k)
#pragma unroll
            for (int m = 0; m < 4; ++m) {
                const float f = xs[grp * 4 + m][k];
                acc[0][m] = fmaf(f, ws[0][col][k], acc[0][m]);
                if constexpr (GLU) acc[1][m] = fmaf(f, ws[1][col][k], acc[1][m]);
            }
        __syncthreads();
    }
    if (n0 + col >= a.n) return;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
        const int item = item_s[grp * 4 + m];
        if (item < 0) continue;
        float y = acc[0][m];
        if constexpr (GLU) y = row_silu<T>(y) * acc[1][m];
        pa_scalar<T>::store(reinterpret_cast<T *>(a.out) + (int64_t)item * a.n + n0 + col, y);
    }
}

int launch_error(const char *what) {
    PA_CHECK_LAUNCH(what);
    return PA_OK;
}

template <int TM, int TN, int WM, int WN, bool GLU> int launch_tiles(const MoeArgs &a, hipStream_t s) {
    constexpr int bm = 16 * TM * WM, bn = 16 * TN * WN, out = GLU ? bn / 2 : bn;
    constexpr size_t lds = (size_t)2 * (bm + bn) * 128 + bm * 4;
    static_assert(lds <= 160 * 1024, "LDS of one compute unit");
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(moe_tile_kernel<TM, TN, WM, WN, GLU>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "pa_moe_product: %s", hipGetErrorString(e));
    }
    const int64_t grid = moe_max_tiles(a.items, a.experts, bm) * ((a.n + out - 1) / out);
    PA_REQUIRE(grid <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    moe_tile_kernel<TM, TN, WM, WN, GLU><<<dim3((unsigned)grid), dim3(64 * WM * WN), lds, s>>>(a);
    return launch_error("pa_moe_product");
}

template <int MT, bool GLU> int launch_stream(const MoeArgs &a, hipStream_t s) {
    const int64_t grid = moe_max_tiles(a.items, a.experts, 16 * MT) * ((a.n + (GLU ? 63 : 127)) / (GLU ? 64 : 128));
    PA_REQUIRE(grid <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    moe_stream_kernel<MT, GLU><<<dim3((unsigned)grid), dim3(256), 0, s>>>(a);
    return launch_error("pa_moe_product");
}

template <typename T, bool GLU> int launch_vector(const MoeArgs &a, hipStream_t s) {
    const int64_t grid = moe_max_tiles(a.items, a.experts, 16) * ((a.n + 63) / 64);
    PA_REQUIRE(grid <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    moe_vector_kernel<T, GLU><<<dim3((unsigned)grid), dim3(256), 0, s>>>(a);
    return launch_error("pa_moe_product");
}

template <bool GLU> int launch_bf16(const MoeArgs &a, hipStream_t s) {
    switch (moe_shape(a.items, a.experts)) {
    case kMoeStream16: return launch_stream<1, GLU>(a, s);
    case kMoeStream32: return launch_stream<2, GLU>(a, s);
    case kMoeStream64: return launch_stream<4, GLU>(a, s);
    case kMoeTile64: return launch_tiles<2, 4, 2, 2, GLU>(a, s);
    default: return launch_tiles<4, 8, 4, 2, GLU>(a, s);
    }
}

}  // namespace

extern "C" int pa_narrow_linear(const void *x, int64_t x_stride, const void *w, float *out, int64_t rows, int n, int k, int dtype,
                                void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && n > 0 && k > 0, "pa_narrow_linear: sizes out of range");
    PA_REQUIRE(x_stride >= k, "pa_narrow_linear: x_stride=%lld is shorter than a row", (long long)x_stride);
    PA_REQUIRE(rows <= 0x7fffffff && (n + 3) / 4 <= 65535, "pa_narrow_linear: too large for one launch");
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_narrow_linear: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x && w && out, "NULL argument");
    NarrowArgs a{x, w, x_stride, out, rows, n, k};
    hipStream_t s = (hipStream_t)stream;
    const unsigned gy = (unsigned)((n + 63) / 64);
    if (dtype == PA_F32) narrow_dot_kernel<float><<<dim3((unsigned)rows, (unsigned)((n + 3) / 4)), dim3(256), 0, s>>>(a);
    else if (k % 8 != 0 || x_stride % 8 != 0 || !pa_aligned16(x) || !pa_aligned16(w))
        narrow_dot_kernel<pa_bf16><<<dim3((unsigned)rows, (unsigned)((n + 3) / 4)), dim3(256), 0, s>>>(a);
    else if (rows <= 2048) narrow_mfma_kernel<1, 8><<<dim3((unsigned)((rows + 15) / 16), gy), dim3(512), 0, s>>>(a);
    else narrow_mfma_kernel<4, 4><<<dim3((unsigned)((rows + 63) / 64), gy), dim3(256), 0, s>>>(a);
    PA_CHECK_LAUNCH("pa_narrow_linear");
    return PA_OK;
}

extern "C" int pa_moe_select(const float *logits, int64_t logits_stride, int64_t rows, int experts, int top, int groups, int keep,
                             int shared, int32_t *ids, float *weights, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && experts > 0 && top > 0 && groups > 0, "pa_moe_select: sizes out of range");
    PA_REQUIRE(experts % groups == 0, "experts=%d are not %d equal groups", experts, groups);
    PA_REQUIRE(keep > 0 && keep <= groups && top <= keep * (experts / groups), "%d experts cannot be chosen from %d of %d groups of %d", top,
               keep, groups, experts / groups);
    if (top > 64 || experts > 1024) return pa_fail(PA_ERR_UNSUPPORTED, "pa_moe_select: top=%d above 64 or experts=%d above 1024", top, experts);
    PA_REQUIRE(logits_stride >= experts + (shared ? 1 : 0), "logits_stride=%lld is shorter than a row", (long long)logits_stride);
    PA_REQUIRE(rows <= 0x7fffffff, "pa_moe_select: rows=%lld is too large for one launch", (long long)rows);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(logits && ids && weights, "NULL argument");
    SelectArgs a{logits, logits_stride, rows, ids, weights, experts, top, groups, keep, shared};
    moe_select_kernel<<<dim3((unsigned)((rows + 3) / 4)), dim3(256), (size_t)4 * (experts + groups) * sizeof(float), (hipStream_t)stream>>>(a);
    PA_CHECK_LAUNCH("pa_moe_select");
    return PA_OK;
}

extern "C" int pa_moe_lists(const int32_t *ids, int64_t rows, int top, int experts, int32_t *counts, int32_t *lists, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && experts > 0 && top > 0, "pa_moe_lists: sizes out of range");
    PA_REQUIRE(rows * top <= 0x7fffffff, "pa_moe_lists: rows=%lld is too large for one launch", (long long)rows);
    PA_REQUIRE(counts && (rows == 0 || (ids && lists)), "NULL argument");
    PA_REQUIRE(pa_aligned16(ids), "ids must be 16-byte aligned");
    moe_lists_kernel<<<dim3((unsigned)experts), dim3(kListThreads), 0, (hipStream_t)stream>>>(ids, rows * top, rows, counts, lists);
    PA_CHECK_LAUNCH("pa_moe_lists");
    return PA_OK;
}

extern "C" int pa_moe_product(const void *x, int64_t x_stride, int items_per_row, const void *w, int64_t w_rows, int w_stride, int k,
                              const int32_t *counts, const int32_t *lists, int64_t rows, int top, int experts, int glu,
                              void *out, int n, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && top > 0 && experts > 0 && items_per_row > 0 && k > 0 && n > 0, "pa_moe_product: sizes out of range");
    PA_REQUIRE(x_stride >= k && w_stride >= k, "pa_moe_product: a stride is shorter than its row");
    PA_REQUIRE(w_rows >= (int64_t)n * (glu ? 2 : 1), "w_rows=%lld are fewer than the outputs need", (long long)w_rows);
    PA_REQUIRE(rows * top <= 0x7fffffff, "pa_moe_product: rows=%lld is too large for one launch", (long long)rows);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_moe_product: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x && w && counts && lists && out, "NULL argument");
    MoeArgs a{x, x_stride, items_per_row, w, w_rows, k, w_stride, n, counts, lists, rows, rows * top, experts, out};
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) return glu ? launch_vector<float, true>(a, s) : launch_vector<float, false>(a, s);
    if (k % 8 != 0 || x_stride % 8 != 0 || w_stride % 64 != 0 || n % 4 != 0 || !pa_aligned16(x) || !pa_aligned16(w) || !pa_aligned16(out))
        return glu ? launch_vector<pa_bf16, true>(a, s) : launch_vector<pa_bf16, false>(a, s);
    return glu ? launch_bf16<true>(a, s) : launch_bf16<false>(a, s);
}
