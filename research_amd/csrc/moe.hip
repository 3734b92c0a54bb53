// Mixture of experts: a narrow product with 32-bit results (router logits), the choice of experts, the list of every
// expert's tokens, and the experts' products over those lists.
//
// An item is (token, place among its chosen experts), numbered token * top + place.  Products write their row of an item
// at the item's number, so nothing is sorted in memory: the lists say which rows an expert reads and writes, and the
// weighted sum over a token's items happens where the result is used (pa_residual_norm).  No counts go through the host.
//
// Product kernels, by how many tokens an expert has on average (moe_plan.h): weights streamed from memory into registers
// for a few; 64 x 128 tiles through a ring of LDS buffers; 256 x 256 tiles by workgroups that stay on their compute unit.
// 32-bit operands have a plain kernel.  The weights' rows are zero-padded to whole 64-element steps; token rows are not
// read past their end.  All products are taken transposed (weight rows as the rows of the result), so that a lane holds
// four consecutive outputs of one item.
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

// 16 RT rows x 16 CT columns per workgroup; its NW waves share the inner dimension.  (k: whole 16-byte vectors)
template <int RT, int CT, int NW> __global__ __launch_bounds__(64 * NW) void narrow_mfma_kernel(const NarrowArgs a) {
    __shared__ float red[NW / 2][RT * CT * 4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    const int64_t r0 = (int64_t)blockIdx.x * 16 * RT;
    const int n0 = blockIdx.y * 16 * CT;
    const uint16_t *xr[RT], *wr[CT];
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const int64_t r = r0 + 16 * t + l16;
        xr[t] = reinterpret_cast<const uint16_t *>(a.x) + (r < a.rows ? r : a.rows - 1) * a.ldx;
    }
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        const int n = n0 + 16 * c + l16;
        wr[c] = reinterpret_cast<const uint16_t *>(a.w) + (int64_t)(n < a.n ? n : a.n - 1) * a.k;
    }
    f4 acc[RT][CT];
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int c = 0; c < CT; ++c) acc[t][c] = f4{0.f, 0.f, 0.f, 0.f};
    // (the four lanes of a row take 32 consecutive bytes each: whole lines, in the same order for both operands.  The next
    // step's rows are on their way while this one's are multiplied.)
    bf8 x[2][RT][2];
    auto fetch = [&](int k0, bf8 (&to)[RT][2]) {
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int k = k0 + 16 * g + 8 * half;
#pragma unroll
            for (int t = 0; t < RT; ++t) to[t][half] = k < a.k ? moe_load(xr[t] + k) : moe_zero();
        }
    };
    auto multiply = [&](int k0, const bf8 (&x)[RT][2]) {
        bf8 w[CT][2];
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int k = k0 + 16 * g + 8 * half;
#pragma unroll
            for (int c = 0; c < CT; ++c) w[c][half] = k < a.k ? moe_load(wr[c] + k) : moe_zero();
        }
#pragma unroll
        for (int half = 0; half < 2; ++half)
#pragma unroll
            for (int c = 0; c < CT; ++c)
#pragma unroll
                for (int t = 0; t < RT; ++t) acc[t][c] = moe_mfma(w[c][half], x[t][half], acc[t][c]);
    };
    constexpr int kStep = 64 * NW;
    fetch(64 * wave, x[0]);
    for (int k0 = 64 * wave; k0 < a.k; k0 += 2 * kStep) {
        fetch(k0 + kStep, x[1]);
        multiply(k0, x[0]);
        if (k0 + kStep >= a.k) break;
        fetch(k0 + 2 * kStep, x[0]);
        multiply(k0 + kStep, x[1]);
    }
#pragma unroll
    for (int step = NW / 2; step >= 1; step /= 2) {
        if (wave >= step && wave < 2 * step) {
#pragma unroll
            for (int t = 0; t < RT; ++t)
#pragma unroll
                for (int c = 0; c < CT; ++c)
#pragma unroll
                    for (int i = 0; i < 4; ++i) red[wave - step][(t * CT + c) * 4 + i][lane] = acc[t][c][i];
        }
        __syncthreads();
        if (wave < step) {
#pragma unroll
            for (int t = 0; t < RT; ++t)
#pragma unroll
                for (int c = 0; c < CT; ++c)
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc[t][c][i] += red[wave][(t * CT + c) * 4 + i][lane];
        }
        __syncthreads();
    }
    if (wave != 0) return;
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const int64_t r = r0 + 16 * t + l16;
        if (r >= a.rows) continue;
#pragma unroll
        for (int c = 0; c < CT; ++c)
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
struct ChooseArgs {
    const float *logits;  // [rows][ld]: the experts', then (shared) one for the shared expert's gate
    int64_t ld, rows;
    const float *correction;  // [experts]: added to the scores where they choose, or NULL
    int32_t *ids;    // [rows][top]
    float *weights;  // [rows][top + 1], the last one the shared expert's; with identity experts one more, the sum of theirs
    int32_t *partial;  // [parts][experts]: how many items of each expert the rows of a part have
    int32_t *counts, *lists;
    int experts, top, groups, keep, shared, part_rows;
    int real;  // experts from here on are identity experts
    int softmax, group_top, renormalize;
};

constexpr float kMoeNone = -3.0e38f;  // stands for minus infinity

__device__ __forceinline__ float moe_wave_max(float top) {
    top = fmaxf(top, pa_dpp<0xB1>(top));   // (the patterns of pa_group_sum)
    top = fmaxf(top, pa_dpp<0x4E>(top));
    top = fmaxf(top, pa_dpp<0x141>(top));
    top = fmaxf(top, pa_dpp<0x140>(top));
    auto lane_of = [&](int l) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, top), l)); };
    return fmaxf(fmaxf(lane_of(0), lane_of(16)), fmaxf(lane_of(32), lane_of(48)));
}

// The largest of NPL values per lane, value i * 64 + lane: its number, the lowest on ties, or -1 when none is above `floor`.
template <int NPL> __device__ __forceinline__ int moe_argmax(const float (&v)[NPL], float floor, float &best) {
    float top = v[0];
#pragma unroll
    for (int i = 1; i < NPL; ++i) top = fmaxf(top, v[i]);
    best = moe_wave_max(top);
    if (!(best > floor)) return -1;
#pragma unroll
    for (int i = 0; i < NPL; ++i) {
        const uint64_t hit = __ballot(v[i] == best);
        if (hit) return i * 64 + __ffsll((unsigned long long)hit) - 1;
    }
    return -1;
}

// Workgroup: a part of the rows, one after the other in each of NW waves.  NPL: experts per lane.
template <int NPL, int NW> __global__ __launch_bounds__(64 * NW) void moe_choose_kernel(const ChooseArgs a) {
    extern __shared__ float choose_lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid / 64;
    int *hist = reinterpret_cast<int *>(choose_lds);
    float *row_s = choose_lds + a.experts * (1 + wave);
    for (int e = tid; e < a.experts; e += 64 * NW) hist[e] = 0;
    __syncthreads();
    const int size = a.experts / a.groups;
    const int64_t first = (int64_t)blockIdx.x * a.part_rows, end = first + a.part_rows < a.rows ? first + a.part_rows : a.rows;
    for (int64_t row = first + wave; row < end; row += NW) {
        const float *logit = a.logits + row * a.ld;
        float s[NPL], weight[NPL];  // what chooses, and what weighs  (a value that is NaN, or not above kMoeNone, cannot be chosen)
        if (a.softmax) {
            float most = kMoeNone, sum = 0.f;
#pragma unroll
            for (int i = 0; i < NPL; ++i) {
                const int e = i * 64 + lane;
                s[i] = e < a.experts ? logit[e] : kMoeNone;
                most = fmaxf(most, s[i]);
            }
            most = moe_wave_max(most);
#pragma unroll
            for (int i = 0; i < NPL; ++i) {
                weight[i] = i * 64 + lane < a.experts ? expf(s[i] - most) : 0.f;
                sum += weight[i];
            }
            sum = pa_group_sum<64>(sum);
#pragma unroll
            for (int i = 0; i < NPL; ++i) weight[i] /= sum;
        } else {
#pragma unroll
            for (int i = 0; i < NPL; ++i) weight[i] = i * 64 + lane < a.experts ? 1.f / (1.f + expf(-logit[i * 64 + lane])) : 0.f;
        }
#pragma unroll
        for (int i = 0; i < NPL; ++i) {
            const int e = i * 64 + lane;
            s[i] = kMoeNone;
            if (e < a.experts) s[i] = weight[i] + (a.correction ? a.correction[e] : 0.f);
            if (!(s[i] > kMoeNone)) s[i] = kMoeNone;
        }
        if (a.keep < a.groups) {
            // (a wave's own part of LDS: its accesses are in order, the compiler must keep them so)
            __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
            for (int i = 0; i < NPL; ++i)
                if (i * 64 + lane < a.experts) row_s[i * 64 + lane] = s[i];
            __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
            __builtin_amdgcn_wave_barrier();
            float value[NPL];  // a group's value: its largest score, or its two largest
            bool able[NPL];
#pragma unroll
            for (int i = 0; i < NPL; ++i) {
                const int g = i * 64 + lane;
                value[i] = kMoeNone;
                able[i] = false;
                if (g >= a.groups) continue;
                float one = kMoeNone, two = kMoeNone;
                for (int e = g * size; e < (g + 1) * size; ++e) {
                    const float x = row_s[e];
                    two = fmaxf(two, fminf(one, x));
                    one = fmaxf(one, x);
                }
                value[i] = a.group_top == 1 || two == kMoeNone ? one : one + two;
            }
            for (int k = 0; k < a.keep; ++k) {
                float best;
                const int g = moe_argmax<NPL>(value, kMoeNone, best);
#pragma unroll
                for (int i = 0; i < NPL; ++i) {
                    if (i * 64 + lane == g) value[i] = kMoeNone;
                    able[i] |= g >= 0 && (i * 64 + lane) / size == g;
                }
            }
#pragma unroll
            for (int i = 0; i < NPL; ++i)
                if (!able[i]) s[i] = kMoeNone;
        }
        float sum = 0.f, mine = 0.f;
        int my_id = -1;
        for (int k = 0; k < a.top; ++k) {
            float best, took = 0.f;
            const int at = moe_argmax<NPL>(s, kMoeNone, best);
            if (at < 0) break;
#pragma unroll
            for (int i = 0; i < NPL; ++i)
                if (i == at / 64) {  // (uniform)
                    took = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, weight[i]), at % 64));
                    if (lane == at % 64) s[i] = kMoeNone;
                }
            sum += took;
            if (lane == k) {
                mine = took;
                my_id = at;
            }
        }
        if (a.renormalize) mine /= sum + 1e-20f;
        // an identity expert's item is in no list: its weight goes to the row's own input
        const bool same = my_id >= a.real;
        const int ld_w = a.top + (a.real < a.experts ? 2 : 1);
        const float own = a.real < a.experts ? pa_group_sum<64>(lane < a.top && same ? mine : 0.f) : 0.f;
        if (lane < a.top) {
            a.ids[row * a.top + lane] = same ? -1 : my_id;
            a.weights[row * ld_w + lane] = same ? 0.f : mine;
            if (my_id >= 0 && !same) atomicAdd(hist + my_id, 1);
        }
        if (lane == 0) {
            a.weights[row * ld_w + a.top] = a.shared == PA_MOE_SHARED_GATED ? 1.f / (1.f + expf(-logit[a.experts])) : a.shared ? 1.f : 0.f;
            if (a.real < a.experts) a.weights[row * ld_w + a.top + 1] = own;
        }
    }
    __syncthreads();
    for (int e = tid; e < a.experts; e += 64 * NW) a.partial[(int64_t)blockIdx.x * a.experts + e] = hist[e];
}

// Workgroup: the same part of the rows.  A thread per expert and stretch of the part's items lists that stretch's items of the
// expert in their order, behind those of the stretches and parts before it.
constexpr int kListThreads = 1024;
__global__ __launch_bounds__(kListThreads) void moe_lists_kernel(const ChooseArgs a) {
    extern __shared__ float choose_lds[];
    __shared__ int sums[2][kListThreads];  // [stretch][expert]: items of earlier parts (a share of them), of the stretch
    int32_t *ids = reinterpret_cast<int32_t *>(choose_lds);
    const int64_t row0 = (int64_t)blockIdx.x * a.part_rows;
    const int rows = (int)(row0 + a.part_rows < a.rows ? a.part_rows : a.rows - row0), n = rows * a.top;
    const int tid = threadIdx.x, stretches = kListThreads / a.experts, e = tid % a.experts, st = tid / a.experts;
    const bool live = st < stretches;
    for (int j = tid; j < n; j += kListThreads) ids[j] = a.ids[row0 * a.top + j];
    int earlier = 0, mine = 0;
    if (live)
        for (int part = st; part < (int)blockIdx.x; part += stretches) earlier += a.partial[(int64_t)part * a.experts + e];
    __syncthreads();
    const int j0 = (int)((int64_t)n * st / stretches), j1 = (int)((int64_t)n * (st + 1) / stretches);
    if (live) {
        for (int j = j0; j < j1; ++j) mine += ids[j] == e;
        sums[0][tid] = earlier;
        sums[1][tid] = mine;
    }
    __syncthreads();
    if (!live) return;
    int64_t at = 0;
    for (int i = 0; i < stretches; ++i) at += sums[0][i * a.experts + e] + (i < st ? sums[1][i * a.experts + e] : 0);
    int32_t *out = a.lists + (int64_t)e * a.rows;
    for (int j = j0; j < j1; ++j)
        if (ids[j] == e && at < a.rows) out[at++] = (int32_t)(row0 * a.top + j);
    if (blockIdx.x == gridDim.x - 1 && st == stretches - 1) a.counts[e] = (int32_t)at;
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

// Wait until at most N of this wave's loads from memory and none of its reads of LDS are under way, then for the workgroup
// (without waiting for the rest of the loads).
template <int N> __device__ __forceinline__ void moe_arrive() {
    asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"(N) : "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}

// WM x WN waves; a wave holds TM tiles of 16 items by TN tiles of 16 weight rows.  GLU: the workgroup's weight rows are half
// gate, half up rows of the same outputs, and a wave's tiles likewise.  A ring of kStages steps of 32 elements in LDS: the
// loads of the steps ahead stay under way over the barriers.
constexpr int kMoeStages = 4, kMoeStep = 32;
template <int TM, int TN, int WM, int WN, bool GLU>
__global__ __launch_bounds__(64 * WM * WN, 2) void moe_tile_kernel(const MoeArgs a) {
    constexpr int kBM = 16 * TM * WM, kBN = 16 * TN * WN, kWaves = WM * WN, kThr = 64 * kWaves;
    constexpr int kLoadsA = kBM / 16 / kWaves, kLoadsB = kBN / 16 / kWaves;  // wave-wide loads of sixteen 64-byte rows
    static_assert(kBM % (16 * kWaves) == 0 && kBN % (16 * kWaves) == 0 && (!GLU || TN % 2 == 0), "whole loads per wave");
    extern __shared__ __align__(16) char lds[];
    // rows of four 16-byte chunks, chunk c of row r at c ^ ((r >> 1) & 3)
    __bf16 *as = reinterpret_cast<__bf16 *>(lds), *bs = as + kMoeStages * kBM * kMoeStep;
    int32_t *item_s = reinterpret_cast<int32_t *>(bs + kMoeStages * kBN * kMoeStep);
    constexpr int kOut = GLU ? kBN / 2 : kBN;  // outputs per workgroup
    const int n_tiles = (a.n + kOut - 1) / kOut;
    const int i = moe_swizzle(blockIdx.x, gridDim.x);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    int expert, m0, count;
    if (!moe_tile(a, i / n_tiles, kBM, lane, expert, m0, count)) return;
    const int n0 = i % n_tiles * kOut;
    // sources of this lane's chunks
    const int r16 = lane / 4, ch = (lane % 4) ^ ((r16 >> 1) & 3);
    const uint16_t *x = reinterpret_cast<const uint16_t *>(a.x), *w = reinterpret_cast<const uint16_t *>(a.w) + expert * a.w_rows * a.kp;
    const uint16_t *pa[kLoadsA], *pb[kLoadsB];
#pragma unroll
    for (int j = 0; j < kLoadsB; ++j) {
        const int r = (wave * kLoadsB + j) * 16 + r16;
        int n = n0 + (GLU ? r % (kBN / 2) : r);
        if (n >= a.n) n = a.n - 1;
        if (GLU && r >= kBN / 2) n += a.n;
        pb[j] = w + (int64_t)n * a.kp + 8 * ch;
    }
#pragma unroll
    for (int j = 0; j < kLoadsA; ++j) {
        const int r = (wave * kLoadsA + j) * 16 + r16;
        int32_t item = m0 + r < count ? a.lists[expert * a.cap + m0 + r] : -1;
        if (item >= a.items) item = -1;
        if (lane % 4 == 0) item_s[r] = item;
        pa[j] = x + (int64_t)((item < 0 ? 0 : item) / a.per_row) * a.ldx;
    }
    const int steps = a.kp / kMoeStep;
    auto fetch = [&](int step) {  // (past the last step: the last one again, so that the number of loads under way is the same)
        const int k0 = (step < steps ? step : steps - 1) * kMoeStep, buf = step % kMoeStages, k = k0 + 8 * ch;
#pragma unroll
        for (int j = 0; j < kLoadsA; ++j)  // (past a row's end: its first elements, against zeros of the weights)
            __builtin_amdgcn_global_load_lds((global_ptr)(pa[j] + (k < a.k ? k : 0)),
                                             (lds_ptr)(as + (buf * kBM + (wave * kLoadsA + j) * 16) * kMoeStep), 16, 0, 0);
#pragma unroll
        for (int j = 0; j < kLoadsB; ++j)
            __builtin_amdgcn_global_load_lds((global_ptr)(pb[j] + k0),
                                             (lds_ptr)(bs + (buf * kBN + (wave * kLoadsB + j) * 16) * kMoeStep), 16, 0, 0);
    };
    const int wm = wave / WN, wn = wave % WN;
    f4 acc[TN][TM];
#pragma unroll
    for (int t = 0; t < TN; ++t)
#pragma unroll
        for (int m = 0; m < TM; ++m) acc[t][m] = f4{0.f, 0.f, 0.f, 0.f};
    // first weight row of the wave's tile t
    auto tile_row = [&](int t) { return GLU ? (t < TN / 2 ? 16 * (wn * TN / 2 + t) : kBN / 2 + 16 * (wn * TN / 2 + t - TN / 2)) : 16 * (wn * TN + t); };
#pragma unroll
    for (int step = 0; step < kMoeStages - 1; ++step) fetch(step);
    const int c8 = (g ^ ((l16 >> 1) & 3)) * 8;
    for (int step = 0; step < steps; ++step) {
        moe_arrive<(kMoeStages - 2) * (kLoadsA + kLoadsB)>();  // this step's tiles are there; the step before has been read
        fetch(step + kMoeStages - 1);
        const __bf16 *ab = as + (step % kMoeStages * kBM + 16 * wm * TM + l16) * kMoeStep + c8;
        const __bf16 *bb = bs + (step % kMoeStages * kBN + l16) * kMoeStep + c8;
        bf8 xa[TM];
#pragma unroll
        for (int m = 0; m < TM; ++m) xa[m] = *reinterpret_cast<const bf8 *>(ab + 16 * m * kMoeStep);
#pragma unroll
        for (int t = 0; t < TN; ++t) {
            const bf8 wb = *reinterpret_cast<const bf8 *>(bb + tile_row(t) * kMoeStep);
#pragma unroll
            for (int m = 0; m < TM; ++m) acc[t][m] = moe_mfma(wb, xa[m], acc[t][m]);
        }
    }
    moe_arrive<0>();  // (nothing may arrive in LDS after the workgroup's end; item_s is complete)
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

// Larger tiles by workgroups that stay: one per compute unit, each takes every so-manieth tile of its die's share.  Two
// buffers of 64 elements; the pipeline runs on over the tiles' borders: while a tile's last steps are multiplied, the next
// tile's first ones are on their way.  Operands run ahead of the products through registers, so that one barrier per step
// (behind the last reads of a buffer) both frees it and admits the other one.
// (At least kStayLeastSteps steps per tile: the next tile's items are looked up in that time.)
constexpr int kStayStep = 64, kStayLeastSteps = 4;
template <int TM, int TN, int WM, int WN, bool GLU>
__global__ __launch_bounds__(64 * WM * WN, 2) void moe_stay_kernel(const MoeArgs a) {
    constexpr int kBM = 16 * TM * WM, kBN = 16 * TN * WN, kWaves = WM * WN;
    constexpr int kLoadsA = kBM / 8 / kWaves, kLoadsB = kBN / 8 / kWaves;  // wave-wide loads of eight 128-byte rows
    constexpr int kOut = GLU ? kBN / 2 : kBN;  // outputs per tile
    constexpr int kRing = 4, kAhead = 2, kGroups = 2 * TN;  // groups of TM products: 32 elements of one weight tile
    constexpr int kStores = TM * (GLU ? TN / 4 : TN / 2);
    static_assert(kBM % (8 * kWaves) == 0 && kBN % (32 * kWaves) == 0 && kBM == 64 * (kWaves / 2) && TN % 4 == 0, "whole loads per wave");
    extern __shared__ __align__(16) char lds[];
    // Rows of eight 16-byte chunks.  Chunk c of item row r is at c ^ ((r >> 1) & 7); a wave reads weight rows four and four,
    // eight apart (below): chunk c of weight row r is at c ^ ((r >> 1 & 1) | (r >> 3 & 3) << 1).
    __bf16 *as = reinterpret_cast<__bf16 *>(lds), *bs = as + 2 * kBM * kStayStep;
    int32_t *item_s = reinterpret_cast<int32_t *>(bs + 2 * kBN * kStayStep);  // [2][kBM], by tile
    int32_t *upto_s = item_s + 2 * kBM;  // [experts]: row tiles of the experts up to this one
    const int n_tiles = (a.n + kOut - 1) / kOut;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l16 = lane & 15, g = lane >> 4, wm = wave / WN, wn = wave % WN;
    int row_tiles = 0;
    for (int e0 = 0; e0 < a.experts; e0 += 64) {  // (every wave, for the total; the first one keeps the sums)
        const int e = e0 + lane, t = e < a.experts ? (a.counts[e] + kBM - 1) / kBM : 0;
        int upto = t;
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const int y = __shfl_up(upto, d, 64);
            if (lane >= d) upto += y;
        }
        if (wave == 0 && e < a.experts) upto_s[e] = row_tiles + upto;
        row_tiles += __builtin_amdgcn_readlane(upto, 63);
    }
    __syncthreads();
    const int64_t total = (int64_t)row_tiles * n_tiles;
    const int die = blockIdx.x % 8, stride = gridDim.x / 8;
    const int end = (int)(total * (die + 1) / 8);
    int tile = (int)(total * die / 8) + blockIdx.x / 8;
    if (tile >= end) return;

    struct Tile {
        int expert, m0, count, n0;
    };
    auto look_up = [&](int tile) {
        Tile t;
        const int rt = tile / n_tiles;
        t.n0 = (tile - rt * n_tiles) * kOut;
        t.expert = 0;
        for (int e0 = 0; e0 < a.experts; e0 += 64) {
            const int e = e0 + lane, upto = e < a.experts ? upto_s[e] : 0x7fffffff;
            const uint64_t past = __ballot(upto > rt);
            if (past) {
                t.expert = e0 + __ffsll((unsigned long long)past) - 1;
                break;
            }
        }
        t.expert = __builtin_amdgcn_readfirstlane(t.expert);
        const int before = t.expert > 0 ? upto_s[t.expert - 1] : 0;
        t.m0 = __builtin_amdgcn_readfirstlane((rt - before) * kBM);
        t.count = a.counts[t.expert];
        return t;
    };
    // The tile's list into LDS: half of the waves bring 64 places each (places past the list's end: its last item).
    auto fetch_items = [&](const Tile &t, int half) {
        if (wave >= kWaves / 2) return;
        const int place = t.m0 + 64 * wave + lane;
        __builtin_amdgcn_global_load_lds((global_ptr)(a.lists + t.expert * a.cap + (place < t.count ? place : t.count - 1)),
                                         (lds_ptr)(item_s + half * kBM + 64 * wave), 4, 0, 0);
    };
    const int r8 = lane / 8;
    struct Sources {  // byte offsets of this lane's rows
        const char *w;
        uint32_t a[kLoadsA], b[kLoadsB];
    };
    auto sources = [&](const Tile &t, int half) {
        Sources s;
        s.w = reinterpret_cast<const char *>(a.w) + t.expert * a.w_rows * a.kp * 2;
#pragma unroll
        for (int j = 0; j < kLoadsB; ++j) {
            const int blk = wave * kLoadsB + j, r = blk * 8 + r8;
            int n = t.n0 + (GLU ? r % (kBN / 2) : r);
            if (n >= a.n) n = a.n - 1;
            if (GLU && r >= kBN / 2) n += a.n;
            s.b[j] = (uint32_t)n * (uint32_t)a.kp * 2u + 16u * ((lane % 8) ^ ((r8 >> 1 & 1) | (blk & 3) << 1));
        }
#pragma unroll
        for (int j = 0; j < kLoadsA; ++j) {
            const uint32_t item = (uint32_t)item_s[half * kBM + (wave * kLoadsA + j) * 8 + r8];
            s.a[j] = (item < a.items ? item / (uint32_t)a.per_row : 0u) * (uint32_t)a.ldx * 2u;
        }
        return s;
    };
    const int steps = a.kp / kStayStep;
    auto fetch = [&](const Sources &s, int step, int buf) {
#pragma unroll
        for (int j = 0; j < kLoadsA; ++j) {  // (past a row's end: its first elements, against zeros of the weights)
            const int blk = wave * kLoadsA + j, k = step * kStayStep + 8 * ((lane % 8) ^ (((blk & 1) << 2) | r8 >> 1));
            __builtin_amdgcn_global_load_lds((global_ptr)(reinterpret_cast<const char *>(a.x) + (s.a[j] + (k < a.k ? 2u * k : 0u))),
                                             (lds_ptr)(as + (buf * kBM + blk * 8) * kStayStep), 16, 0, 0);
        }
#pragma unroll
        for (int j = 0; j < kLoadsB; ++j)
            __builtin_amdgcn_global_load_lds((global_ptr)(s.w + (s.b[j] + 2u * step * kStayStep)),
                                             (lds_ptr)(bs + (buf * kBN + (wave * kLoadsB + j) * 8) * kStayStep), 16, 0, 0);
    };
    // Product tile t of a wave takes the weight rows 32 (t / 2) + 8 (row / 4) + 4 (t & 1) + row % 4 of its share, so that a
    // lane's results of two tiles are eight consecutive outputs.  (GLU: the first half of the tiles are gate rows.)
    auto tile_row = [&](int t) {
        const int q = GLU ? t % (TN / 2) : t;
        return (GLU && t >= TN / 2 ? kBN / 2 : 0) + 16 * wn * (GLU ? TN / 2 : TN) + 32 * (q / 2) + 4 * (q & 1);
    };
    const int a_swz = (l16 >> 1) & 7, b_swz = (l16 >> 1 & 1) | (l16 >> 2) << 1;
    const __bf16 *ab = as + (16 * wm * TM + l16) * kStayStep, *bb = bs + (8 * (l16 / 4) + l16 % 4) * kStayStep;
    auto a_tile = [&](int buf, int kk, int m) {
        return *reinterpret_cast<const bf8 *>(ab + (buf * kBM + 16 * m) * kStayStep + 8 * ((4 * kk + g) ^ a_swz));
    };
    auto b_tile = [&](int buf, int group) {
        return *reinterpret_cast<const bf8 *>(bb + (buf * kBN + tile_row(group % TN)) * kStayStep + 8 * ((4 * (group / TN) + g) ^ b_swz));
    };

    Tile now = look_up(tile), next = now;
    fetch_items(now, 0);
    moe_arrive<0>();
    Sources src = sources(now, 0);
    int half = 0;  // of item_s
    fetch(src, 0, 0);
    fetch(src, 1, 1);
    f4 acc[TN][TM];
    bf8 xa[2][TM], wb[kRing];
    moe_arrive<kLoadsA + kLoadsB>();
#pragma unroll
    for (int m = 0; m < TM; ++m) xa[0][m] = a_tile(0, 0, m);
#pragma unroll
    for (int t = 0; t < kAhead; ++t) wb[t] = b_tile(0, t);
    // One step from buffer `buf`.  Behind its last reads: the other buffer's tiles have come (`stores`: the last tile's results,
    // which are younger, need not have been written), every wave is through with this one, and step `far` is sent for.
    auto run = [&](int buf, int far, bool stores) {
#pragma unroll
        for (int q = 0; q < kGroups; ++q) {
            if (q == kGroups - kAhead) {
                if (stores) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kStores) : "memory");
                else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
                asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                __builtin_amdgcn_s_barrier();
                asm volatile("" ::: "memory");
                fetch(src, far, buf);
            }
            const int to = q + kAhead;
            wb[to % kRing] = to < kGroups ? b_tile(buf, to) : b_tile(buf ^ 1, to - kGroups);
            if (q == TN / 2) {  // the second half's items
#pragma unroll
                for (int m = 0; m < TM; ++m) xa[1][m] = a_tile(buf, 1, m);
            }
            if (q == kGroups - kAhead) {  // the next step's
#pragma unroll
                for (int m = 0; m < TM; ++m) xa[0][m] = a_tile(buf ^ 1, 0, m);
            }
#pragma unroll
            for (int m = 0; m < TM; ++m) acc[q % TN][m] = moe_mfma(wb[q % kRing], xa[q / TN][m], acc[q % TN][m]);
        }
    };
    const __amdgpu_buffer_rsrc_t dst = __builtin_amdgcn_make_buffer_rsrc(a.out, 0, (int)(uint32_t)(a.items * a.n * 2), 0x00020000);
    int buf = 0;
    bool first = true;
    for (;;) {
#pragma unroll
        for (int t = 0; t < TN; ++t)
#pragma unroll
            for (int m = 0; m < TM; ++m) acc[t][m] = f4{0.f, 0.f, 0.f, 0.f};
        const int tile_next = tile + stride;
        const bool more = tile_next < end;
        for (int step = 0; step < steps; ++step) {
            // (the next tile's items came before the wait of step 1, in every wave before its barrier)
            if (step == steps - 2 && more) src = sources(next, half ^ 1);
            run(buf, step + 2 < steps ? step + 2 : step + 2 - steps, step == 0 && !first);
            buf ^= 1;
            if (step == 0 && more) {  // (every wave is past its use of the other half of item_s)
                next = look_up(tile_next);
                fetch_items(next, half ^ 1);
            }
        }
#pragma unroll
        for (int m = 0; m < TM; ++m) {  // (as many stores in every wave; those of missing items or outputs go past the end)
            const int r = 16 * (wm * TM + m) + l16;
            const uint32_t item = (uint32_t)item_s[half * kBM + r];
            const bool live = now.m0 + r < now.count && item < a.items;
#pragma unroll
            for (int t = 0; t < (GLU ? TN / 2 : TN); t += 2) {
                const int n = now.n0 + 16 * wn * (GLU ? TN / 2 : TN) + 16 * t + 8 * g;
                uint32_t p[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const f4 y = acc[t + i / 2][m];
                    if constexpr (GLU) {
                        const f4 u = acc[t + i / 2 + TN / 2][m];
                        p[i] = moe_glu2(y[2 * i % 4], u[2 * i % 4], y[2 * i % 4 + 1], u[2 * i % 4 + 1]);
                    } else {
                        p[i] = row_pack_bf16(y[2 * i % 4], y[2 * i % 4 + 1]);
                    }
                }
                typedef uint32_t u4 __attribute__((ext_vector_type(4)));
                __builtin_amdgcn_raw_buffer_store_b128(u4{p[0], p[1], p[2], p[3]}, dst,
                                                       live && n < a.n ? (item * (uint32_t)a.n + n) * 2u : 0xfffffff0u, 0, 0);
            }
        }
        if (!more) break;
        first = false;
        tile = tile_next;
        now = next;
        half ^= 1;
    }
    moe_arrive<0>();  // (nothing may arrive in LDS after the workgroup's end)
}

// One or two items per expert: every wave streams two tiles of 16 weight rows (GLU: the gate and up rows of the same outputs)
// past a tile of 16 items, without LDS.
template <bool GLU> __global__ __launch_bounds__(256) void moe_stream_kernel(const MoeArgs a) {
    constexpr int kOut = GLU ? 64 : 128;  // outputs per workgroup
    const int n_tiles = (a.n + kOut - 1) / kOut;
    const int i = moe_swizzle(blockIdx.x, gridDim.x);
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int l16 = lane & 15, g = lane >> 4;
    int expert, m0, count;
    if (!moe_tile(a, i / n_tiles, 16, lane, expert, m0, count)) return;
    const int n0 = i % n_tiles * kOut + wave * (GLU ? 16 : 32);
    if (n0 >= a.n) return;
    const uint16_t *w = reinterpret_cast<const uint16_t *>(a.w) + expert * a.w_rows * a.kp + 16 * g;
    auto w_row = [&](int n) { return w + (int64_t)(n < a.n ? n : a.n - 1) * a.kp; };
    const uint16_t *w0 = w_row(n0 + l16), *w1 = GLU ? w0 + (int64_t)a.n * a.kp : w_row(n0 + 16 + l16);
    int item = m0 + l16 < count ? a.lists[expert * a.cap + m0 + l16] : -1;
    if (item >= a.items) item = -1;
    const uint16_t *x = reinterpret_cast<const uint16_t *>(a.x) + (int64_t)((item < 0 ? 0 : item) / a.per_row) * a.ldx;
    f4 y = f4{0.f, 0.f, 0.f, 0.f}, z = y;
    // The next steps' operands are on their way in registers.  (The four lanes of a row take 32 consecutive bytes each: whole
    // lines, in the same order for both operands.)
    constexpr int kAhead = 4;
    bf8 wv[kAhead][2][2], xv[kAhead][2];
    const int steps = a.kp / 64;
    auto fetch = [&](int step, bf8 (&w)[2][2], bf8 (&v)[2]) {
        if (step >= steps) return;
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int k0 = step * 64 + 8 * half, k = k0 + 16 * g;
            w[half][0] = moe_load(w0 + k0);
            w[half][1] = moe_load(w1 + k0);
            v[half] = moe_load(x + (k < a.k ? k : 0));
        }
    };
#pragma unroll
    for (int j = 0; j < kAhead; ++j) fetch(j, wv[j], xv[j]);
    for (int step0 = 0; step0 < steps; step0 += kAhead) {
#pragma unroll
        for (int j = 0; j < kAhead; ++j) {
            if (step0 + j >= steps) break;
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                y = moe_mfma(wv[j][half][0], xv[j][half], y);
                z = moe_mfma(wv[j][half][1], xv[j][half], z);
            }
            fetch(step0 + j + kAhead, wv[j], xv[j]);
        }
    }
    if (item < 0) return;
    uint16_t *row = reinterpret_cast<uint16_t *>(a.out) + (int64_t)item * a.n;
    const int n = n0 + 4 * g;
    if constexpr (GLU) {
        if (n < a.n) *reinterpret_cast<uint2 *>(row + n) = make_uint2(moe_glu2(y[0], z[0], y[1], z[1]), moe_glu2(y[2], z[2], y[3], z[3]));
    } else {
        if (n < a.n) *reinterpret_cast<uint2 *>(row + n) = make_uint2(row_pack_bf16(y[0], y[1]), row_pack_bf16(y[2], y[3]));
        if (n + 16 < a.n) *reinterpret_cast<uint2 *>(row + n + 16) = make_uint2(row_pack_bf16(z[0], z[1]), row_pack_bf16(z[2], z[3]));
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
    constexpr size_t lds = (size_t)kMoeStages * (bm + bn) * kMoeStep * 2 + bm * 4;
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

int moe_cus() {
    static int cached[64];
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return 256;
    int n = __atomic_load_n(&cached[dev], __ATOMIC_RELAXED);
    if (n == 0) {
        if (hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0) n = 256;
        __atomic_store_n(&cached[dev], n, __ATOMIC_RELAXED);
    }
    return n;
}

template <bool GLU> int launch_stay(const MoeArgs &a, hipStream_t s) {
    constexpr int TM = 4, TN = 8, WM = 4, WN = 2, bm = 16 * TM * WM, bn = 16 * TN * WN;
    const size_t lds = (size_t)2 * (bm + bn) * kStayStep * 2 + (size_t)(2 * bm + a.experts) * 4;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(moe_stay_kernel<TM, TN, WM, WN, GLU>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "pa_moe_product: %s", hipGetErrorString(e));
    const int64_t tiles = moe_max_tiles(a.items, a.experts, bm) * ((a.n + (GLU ? bn / 2 : bn) - 1) / (GLU ? bn / 2 : bn));
    PA_REQUIRE(tiles <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    const unsigned grid = (unsigned)((tiles < moe_cus() ? tiles : moe_cus()) + 7) / 8 * 8;  // (whole rounds over the dies)
    moe_stay_kernel<TM, TN, WM, WN, GLU><<<dim3(grid), dim3(64 * WM * WN), lds, s>>>(a);
    return launch_error("pa_moe_product");
}

template <bool GLU> int launch_stream(const MoeArgs &a, hipStream_t s) {
    const int64_t grid = moe_max_tiles(a.items, a.experts, 16) * ((a.n + (GLU ? 63 : 127)) / (GLU ? 64 : 128));
    PA_REQUIRE(grid <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    moe_stream_kernel<GLU><<<dim3((unsigned)grid), dim3(256), 0, s>>>(a);
    return launch_error("pa_moe_product");
}

template <typename T, bool GLU> int launch_vector(const MoeArgs &a, hipStream_t s) {
    const int64_t grid = moe_max_tiles(a.items, a.experts, 16) * ((a.n + 63) / 64);
    PA_REQUIRE(grid <= 0x7fffffff, "pa_moe_product: too many tiles for one launch");
    moe_vector_kernel<T, GLU><<<dim3((unsigned)grid), dim3(256), 0, s>>>(a);
    return launch_error("pa_moe_product");
}

template <bool GLU> int launch_bf16(const MoeArgs &a, hipStream_t s) {
    const MoeShape shape = moe_shape(a.items, a.experts);
    if (shape == kMoeStream) return launch_stream<GLU>(a, s);
    // (32-bit offsets into the rows of x, one expert's weights and the outputs, 16-byte stores)
    const int64_t most = 0xffffff00ll, x_rows = a.items / a.per_row;
    const bool stay = a.kp >= kStayLeastSteps * kStayStep && a.n % 8 == 0 && a.experts <= 1024 && x_rows * a.ldx * 2 <= most &&
                      a.w_rows * a.kp * 2 <= most && a.items * a.n * 2 <= most;
    return shape == kMoeTile256 && stay ? launch_stay<GLU>(a, s) : launch_tiles<2, 4, 2, 2, GLU>(a, s);
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
    if (dtype == PA_F32) narrow_dot_kernel<float><<<dim3((unsigned)rows, (unsigned)((n + 3) / 4)), dim3(256), 0, s>>>(a);
    else if (k % 8 != 0 || x_stride % 8 != 0 || !pa_aligned16(x) || !pa_aligned16(w))
        narrow_dot_kernel<pa_bf16><<<dim3((unsigned)rows, (unsigned)((n + 3) / 4)), dim3(256), 0, s>>>(a);
    else {
        const int tiles = (n + 15) / 16;
        const bool five = tiles % 4 == 1 && tiles > 1;  // (one row more than whole tiles of 64: the gate of a shared expert)
        const unsigned gx = (unsigned)((rows + 15) / 16), gx4 = (unsigned)((rows + 63) / 64), gy = (unsigned)((tiles + (five ? 4 : 3)) / (five ? 5 : 4));
        if (rows <= 1024) narrow_mfma_kernel<1, 1, 8><<<dim3(gx, (unsigned)tiles), dim3(512), 0, s>>>(a);
        else if (five) narrow_mfma_kernel<4, 5, 4><<<dim3(gx4, gy), dim3(256), 0, s>>>(a);
        else narrow_mfma_kernel<4, 4, 4><<<dim3(gx4, gy), dim3(256), 0, s>>>(a);
    }
    PA_CHECK_LAUNCH("pa_narrow_linear");
    return PA_OK;
}

extern "C" size_t pa_moe_workspace_bytes(int64_t rows, int experts, int top) {
    if (rows < 0 || experts <= 0 || top <= 0) return 0;
    return (size_t)moe_parts(rows, top) * experts * sizeof(int32_t);
}

extern "C" int pa_moe_choose(const float *logits, int64_t logits_stride, int64_t rows, int experts, int identity, int top, int groups,
                             int keep, int shared, int scores, int group_top, int renormalize, const float *correction, int32_t *ids,
                             float *weights, int32_t *counts, int32_t *lists, void *workspace, size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && experts > 0 && identity >= 0 && top > 0 && groups > 0, "pa_moe_choose: sizes out of range");
    const int all = experts + identity;
    PA_REQUIRE(all % groups == 0, "experts=%d are not %d equal groups", all, groups);
    PA_REQUIRE(keep > 0 && keep <= groups && top <= keep * (all / groups), "%d experts cannot be chosen from %d of %d groups of %d", top,
               keep, groups, all / groups);
    if (top > 64 || all > 1024) return pa_fail(PA_ERR_UNSUPPORTED, "pa_moe_choose: top=%d above 64 or experts=%d above 1024", top, all);
    PA_REQUIRE(scores == PA_MOE_SIGMOID || scores == PA_MOE_SOFTMAX, "scores=%d is unknown", scores);
    PA_REQUIRE(group_top == 1 || group_top == 2, "group_top=%d is not 1 or 2", group_top);
    PA_REQUIRE(shared >= PA_MOE_NO_SHARED && shared <= PA_MOE_SHARED, "shared=%d is unknown", shared);
    PA_REQUIRE(logits_stride >= all + (shared == PA_MOE_SHARED_GATED ? 1 : 0), "logits_stride=%lld is shorter than a row", (long long)logits_stride);
    PA_REQUIRE(rows * top <= 0x7fffffff, "pa_moe_choose: rows=%lld is too large for one launch", (long long)rows);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(logits && ids && weights && counts && lists, "NULL argument");
    if (!workspace || workspace_bytes < pa_moe_workspace_bytes(rows, all, top))
        return pa_fail(PA_ERR_WORKSPACE, "pa_moe_choose: workspace of %zu bytes, %zu needed", workspace_bytes,
                       pa_moe_workspace_bytes(rows, all, top));
    const int part_rows = moe_part_rows(rows, top);
    ChooseArgs a{logits, logits_stride, rows, correction, ids, weights, (int32_t *)workspace, counts, lists, all, top, groups, keep, shared,
                 part_rows, experts, scores == PA_MOE_SOFTMAX, group_top, renormalize};
    const dim3 grid((unsigned)moe_parts(rows, top));
    auto lds = [&](int waves) { return (size_t)(1 + waves) * all * sizeof(float); };
    hipStream_t s = (hipStream_t)stream;
    if (all <= 64) moe_choose_kernel<1, 16><<<grid, dim3(1024), lds(16), s>>>(a);
    else if (all <= 128) moe_choose_kernel<2, 16><<<grid, dim3(1024), lds(16), s>>>(a);
    else if (all <= 256) moe_choose_kernel<4, 16><<<grid, dim3(1024), lds(16), s>>>(a);
    else moe_choose_kernel<16, 4><<<grid, dim3(256), lds(4), s>>>(a);
    PA_CHECK_LAUNCH("pa_moe_choose");
    moe_lists_kernel<<<grid, dim3(kListThreads), (size_t)part_rows * top * sizeof(int32_t), s>>>(a);
    PA_CHECK_LAUNCH("pa_moe_choose (lists)");
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
