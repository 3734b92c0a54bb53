// Portions of prompts of attention with mixed heads on the matrix cores (16-bit pools, keys and values of up to 128, up to 32
// heads).
//
// The first kernel leaves every row's and head's sum: a wave owns 32 rows of one head, a workgroup four (row block, head) pairs
// of one kv head, which share tiles of 64 keys in LDS (as in scored_prefill.hip, without values).  The second one makes the
// scores again, for all heads at once: a workgroup owns 16 rows and 16 out heads, its eight waves have their own heads' queries
// and two out heads' accumulators in registers.  Per tile of 32 keys
//   1. S^T = K Q^T leaves a lane four keys of one row per head; the weights go to LDS, all heads of a (key, row) pair side by
//      side, as two bf16 terms;
//   2. T times these, the pairs of four keys per wave, and back to LDS as weights of (out head, row), keys side by side;
//   3. O^T += V^T W^T per out head, V by transposing reads from the wave's own part of LDS.
// The next tile's keys and values are on their way in registers.  Distance biases of a head are one logarithm per lane and
// tile, spread by LDS.
#include "linear_tiles.h"
#include "prefill_mfma.h"
#include "talking.h"

namespace {

using namespace pa_decode_detail;

constexpr float kTpSlack = 8.f;  // log2 of the factor by which a row's reference maximum may lag

__device__ __forceinline__ void tp_own_lds() {  // a wave's own part of LDS: its writes before its reads
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
}

// ------------------------------------------------------------------ sums
constexpr int kTsKeys = 64;
template <int DK> __global__ __launch_bounds__(256, 2) void talk_sums_kernel(const TalkArgs a) {
    using M = Mfma16<pa_bf16>;
    using X8 = M::x8;
    constexpr int KS = DK / 16, NK = kTsKeys * DK / 8 / 256, kPitch = DK + 8;
    __shared__ __align__(16) uint16_t ks[kTsKeys * kPitch];
    __shared__ float biases[4][2][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), half = lane >> 5, col = lane & 31;
    const int kvh = blockIdx.y, b = blockIdx.x;
    ScoredPortion p;
    if (!scored_portion(a, b, p)) return;
    const int n_tasks = (p.n + 31) / 32 * a.n_rep;
    const int group = gridDim.z - 1 - blockIdx.z;  // (the rows with the most keys first)
    if (group * 4 >= n_tasks) return;
    const int task = group * 4 + wave, last_task = min(n_tasks, group * 4 + 4) - 1;
    const bool live = task < n_tasks;
    const int row0 = (live ? task / a.n_rep : 0) * 32, h = kvh * a.n_rep + (live ? task % a.n_rep : 0);
    const int row = row0 + col, wave_hi = p.pos0 + min(row0 + 32, p.n);
    const int wg_hi = p.pos0 + min(last_task / a.n_rep * 32 + 32, p.n);
    const float plain = a.scale * kScoredLog2e, size = a.size ? a.size[h] : 0.f, rate = a.rate ? a.rate[h] : 0.f;
    X8 q[KS];
    {
        const uint16_t *src = reinterpret_cast<const uint16_t *>(a.q1) + (p.row0 + min(row, p.n - 1)) * a.q1_row + h * a.q1_head;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int d = 16 * k + 8 * half;
            q[k] = __builtin_bit_cast(X8, d < a.n1 ? *reinterpret_cast<const uint4 *>(src + d) : make_uint4(0, 0, 0, 0));
        }
    }
    // the row's reference m, which the products start from (as -m / plain), and the sum of 2^(score - m)
    float m = 0.f, l = 0.f;
    const float unplain = 1.f / plain;
    f32x16 start;
#pragma unroll
    for (int i = 0; i < 16; ++i) start[i] = 0.f;
    const int32_t *table = a.bt + b * a.bt_stride;
    const uint16_t *kp = reinterpret_cast<const uint16_t *>(a.k) + (int64_t)kvh * a.k_dim;
    const int64_t k_tok = (int64_t)a.hkv * a.k_dim;
    auto id_of = [&](int k0) { return talk_block_id(a, table, min(k0 + lane, wg_hi - 1)); };
    scored_u4 kr[NK];
    auto fetch = [&](int id, int k0) {
        const int slots = talk_slot_of(a, id, k0 + lane, wg_hi);
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            const int c = tid + 256 * n, s = __shfl(slots, c / (DK / 8), 64), e = c % (DK / 8) * 8;
            kr[n] = scored_load16(kp + s * k_tok + e, s >= 0 && e < a.n1);
        }
    };
    fetch(id_of(0), 0);
    int id = id_of(kTsKeys);
    for (int k0 = 0; k0 < wg_hi; k0 += kTsKeys) {
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            const int c = tid + 256 * n;
            *reinterpret_cast<scored_u4 *>(ks + c / (DK / 8) * kPitch + c % (DK / 8) * 8) = kr[n];
        }
        __syncthreads();
        if (k0 + kTsKeys < wg_hi) {
            fetch(id, k0 + kTsKeys);
            id = id_of(k0 + 2 * kTsKeys);
        }
        if (live && k0 < wave_hi) {  // distances p.pos0 + row0 + i - k of i < 32 and each half's 32 keys, from their smallest
#pragma unroll
            for (int sub = 0; sub < 2; ++sub)
                biases[wave][sub][lane] = talk_masked_bias(size, rate, p.pos0 + row0 - (k0 + 32 * sub + 31) + lane);
            tp_own_lds();
        }
#pragma unroll
        for (int sub = 0; sub < 2; ++sub) {
            const int kb = k0 + 32 * sub;  // (uniform per wave)
            if (!live || kb >= wave_hi) continue;
            f32x16 s = start;
#pragma unroll
            for (int k = 0; k < KS; ++k)
                s = M::mma(__builtin_bit_cast(X8, *reinterpret_cast<const uint4 *>(ks + (32 * sub + col) * kPitch + 16 * k + 8 * half)), q[k], s);
            // element i: key kb + 8 (i / 4) + 4 half + i % 4
            const float *bp = biases[wave][sub] + col + 31 - 4 * half;
#pragma unroll
            for (int i = 0; i < 16; ++i) s[i] = fmaf(s[i], plain, bp[-(8 * (i >> 2) + (i & 3))]);
            float top = fmaxf(s[0], s[1]);
#pragma unroll
            for (int i = 2; i < 16; ++i) top = fmaxf(top, s[i]);
            // (every lane has a reference of its own; it follows when a score is far above it, or the first ones all far below)
            if (__ballot(top > kTpSlack || (l == 0.f && top > 0.5f * kScoredNone && top < -kTpSlack)) != 0) {
                const float by = top > kTpSlack || (l == 0.f && top > 0.5f * kScoredNone) ? top : 0.f;
                l *= __builtin_amdgcn_exp2f(-by);
                m += by;
#pragma unroll
                for (int i = 0; i < 16; ++i) {
                    s[i] -= by;
                    start[i] = -m * unplain;
                }
            }
#pragma unroll
            for (int i = 0; i < 16; i += 2) l += __builtin_amdgcn_exp2f(s[i]) + __builtin_amdgcn_exp2f(s[i + 1]);
        }
        __syncthreads();
    }
    // (a lane that saw no key has nothing to say)
    if (l == 0.f) m = kScoredNone;
    const float other = __shfl_xor(m, 32, 64), top = fmaxf(m, other);
    l *= __builtin_amdgcn_exp2f(m - top);
    l += __shfl_xor(l, 32, 64);
    if (live && row < p.n && half == 0) a.lse[(p.row0 + row) * a.heads + h] = top + __builtin_amdgcn_logf(l);
}

// ------------------------------------------------------------------ mixed weights times values
constexpr int kTmRows = 16, kTmKeys = 32, kTmWaves = 8, kTmThreads = 64 * kTmWaves;
constexpr int kTmOut = 2 * kTmWaves;  // out heads of a workgroup, two per wave

// HW: heads per wave, 2 or 4.  NG: kv heads of the out heads, whose values are staged by the whole workgroup (0: each wave
// stages its own).  With two heads per wave the keys of up to NG kv heads are staged as well.
template <int D, int HW, int NG> struct TmTile {
    static constexpr int heads = kTmWaves * HW, kPitch = D + 8, vPitch = NG ? D + 16 : D + 8;
    static constexpr bool keys = NG > 0 && HW == 2;
    static constexpr int pair = 4 * heads;  // bytes of a (key, row) pair: both terms of all heads
    static constexpr int pBytes = kTmKeys * kTmRows * pair, wBytes = kTmOut * kTmRows * kTmKeys * 2, kTile = kTmKeys * kPitch, vTile = kTmKeys * vPitch + (NG ? 3 * 64 : 0);
    // (a transposing read takes four rows of four sets eight apart)
    static constexpr __device__ int vRow(int row) { return row * vPitch + (NG ? row / 8 * 64 : 0); }
    static constexpr int vBytes = (NG ? NG : kTmWaves) * vTile * 2, kBytes = keys ? NG * kTile * 2 : 0;
    static constexpr int biasFloats = HW * 48;
    static constexpr size_t bytes = (size_t)pBytes + wBytes + vBytes + kBytes + kTmWaves * biasFloats * 4;
};

// D: keys and values padded to 64 or 128; FULL: they fill it.  NG > 0: a wave's heads share a kv head, and so do its out heads.
template <int D, int HW, bool FULL, int NG> __global__ __launch_bounds__(kTmThreads) void talk_mix_kernel(const TalkArgs a) {
    using L = TmTile<D, HW, NG>;
    constexpr bool SAME = NG > 0;
    constexpr int HP = L::heads, KS = D / 32, ET = D / 16;
    constexpr int kPer = D / 8, kTile = kTmKeys * kPer;                     // 16-byte pieces of a row, of a kv head's tile
    constexpr int NV = SAME ? NG * kTile / kTmThreads : kTile / 64, NK = L::keys ? NV : 2 * KS;
    extern __shared__ __align__(16) char tm_lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    char *w_s = tm_lds + L::pBytes;
    __bf16 *v_all = reinterpret_cast<__bf16 *>(w_s + L::wBytes), *k_s = v_all + L::vBytes / 2;
    float *biases = reinterpret_cast<float *>(w_s + L::wBytes + L::vBytes + L::kBytes) + wave * L::biasFloats;
    const int b = blockIdx.x;
    ScoredPortion p;
    if (!scored_portion(a, b, p)) return;
    const int row0 = (int)(gridDim.y - 1 - blockIdx.y) * kTmRows;  // (the rows with the most keys first)
    if (row0 >= p.n) return;
    const int row = row0 + l16, first_pos = p.pos0 + row0, end = p.pos0 + min(row0 + kTmRows, p.n);
    const float plain = a.scale * kScoredLog2e;
    const int head0 = wave * HW, out0 = blockIdx.z * kTmOut, own0 = out0 + 2 * wave;  // the wave's heads and out heads
    auto kv_of = [&](int h) { return min(h, a.heads - 1) / a.n_rep; };
    // T in the pairs' k order (terms of 32 heads, or both of 16): out head out0 + l16; the second term of T meets the first of
    // the weights only
    bf8 t_hi, t_lo;
    bool t_rest;  // (a matrix stored in 16 bits has no second term)
    {
        LaSplit sp;
        bool exact = true;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            float x[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const int turned = HW == 4 ? j ^ (2 * (wave & 1)) : j ^ (wave & 3);  // (as the weights of this wave's keys lie)
                const int out = out0 + l16, in = (8 * g + 2 * turned + e) % HP;
                x[e] = out < a.heads && in < a.heads ? a.talk[(int64_t)out * a.heads + in] : 0.f;
            }
            la_split2(x[0], x[1], sp.hi[j], sp.lo[j]);
            exact = exact && sp.lo[j] == 0;
            if (HP == 16 && g >= 2) sp.lo[j] = 0;
        }
        t_hi = sp.high();
        t_lo = sp.low();
        t_rest = __ballot(!exact) != 0;
    }
    bf8 q[HW][KS];
    float lse[HW], size[HW], rate[HW];
    f4 start[HW];  // two heads per wave: the products start from -lse
    {
        const int64_t mem_row = p.row0 + min(row, p.n - 1);
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            const int h = min(head0 + i, a.heads - 1);
            const uint16_t *src = reinterpret_cast<const uint16_t *>(a.q1) + mem_row * a.q1_row + h * a.q1_head;
#pragma unroll
            for (int k = 0; k < KS; ++k) q[i][k] = __builtin_bit_cast(bf8, scored_load16(src + 32 * k + 8 * g, 32 * k + 8 * g < a.n1));
            lse[i] = row < p.n && head0 + i < a.heads ? a.lse[mem_row * a.heads + h] : -kScoredNone;  // (no head, no row: no weight)
            size[i] = a.size ? a.size[h] : 0.f;
            rate[i] = a.rate ? a.rate[h] : 0.f;
            const float from = HW == 2 ? -lse[i] / plain : 0.f;
            start[i] = f4{from, from, from, from};
        }
    }
    f4 o[2][ET];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int t = 0; t < ET; ++t) o[i][t] = f4{0.f, 0.f, 0.f, 0.f};

    const int32_t *table = a.bt + b * a.bt_stride;
    const uint32_t k_tok = (uint32_t)(a.hkv * a.k_dim), v_tok = (uint32_t)(a.hkv * a.v_dim);
    const int vreal = (a.vdim + 7) / 8 * 8;
    // the kv heads that are staged: from the first of the out heads, from the first of all
    const int v_kv0 = kv_of(out0);
    __bf16 *v_s = v_all + (SAME ? kv_of(own0) - v_kv0 : wave) * L::vTile;
    // Block and pool row of the key that this thread stages (values staged by all: the piece of a tile; else key lane % 32); past
    // the last key: the last one's, which nothing weighs.
    const int my_row = SAME ? tid % kTile / kPer : lane & 31;
    auto key_of = [&](int k0) { return min(k0 + my_row, end - 1); };
    auto id_of = [&](int k0) { return talk_block_id(a, table, key_of(k0)); };
    auto slot_of = [&](int id, int k0) { return max(talk_slot_of(a, id, key_of(k0), end), 0); };
    scored_u4 kr[NK], vr[NV];
    // staged by the workgroup: piece tid + 512 n is of kv head (tid + 512 n) / kTile, the thread's own row
    auto stage_from = [&](const void *pool, int slot, uint32_t tok, int head_dim, int kv_first, int real, scored_u4 *to) {
        const uint16_t *src = reinterpret_cast<const uint16_t *>(pool) + (uint64_t)(uint32_t)slot * tok + tid % kPer * 8;
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const uint16_t *at = src + min(kv_first + (tid + kTmThreads * n) / kTile, a.hkv - 1) * head_dim;
            to[n] = FULL ? *reinterpret_cast<const scored_u4 *>(at) : scored_load16(at, tid % kPer * 8 < real);
        }
    };
    auto stage_to = [&](__bf16 *tiles, int tile, int row_at, const scored_u4 *from) {
#pragma unroll
        for (int n = 0; n < NV; ++n) *reinterpret_cast<scored_u4 *>(tiles + (tid + kTmThreads * n) / kTile * tile + row_at + tid % kPer * 8) = from[n];
    };
    // straight to operands: keys 16 kb + l16 of one kv head (slots: of key lane % 32)
    auto direct_k = [&](int kv, int slots) {
        if constexpr (!L::keys) {
#pragma unroll
            for (int kb = 0; kb < 2; ++kb) {
                const uint16_t *src = reinterpret_cast<const uint16_t *>(a.k) + (uint64_t)(uint32_t)__shfl(slots, 16 * kb + l16, 64) * k_tok + kv * a.k_dim + 8 * g;
#pragma unroll
                for (int k = 0; k < KS; ++k) kr[kb * KS + k] = FULL ? *reinterpret_cast<const scored_u4 *>(src + 32 * k) : scored_load16(src + 32 * k, 32 * k + 8 * g < a.n1);
            }
        }
    };
    auto fetch_k = [&](int slots, int near) {  // (near: the slots of keys lane % 32)
        if constexpr (L::keys) stage_from(a.k, slots, k_tok, a.k_dim, 0, a.n1, kr);
        else direct_k(kv_of(head0), near);
    };
    auto own_v = [&](int kv, int slots) {
        if constexpr (!SAME) {
#pragma unroll
            for (int n = 0; n < NV; ++n) {
                const uint16_t *src = reinterpret_cast<const uint16_t *>(a.v) + (uint64_t)(uint32_t)__shfl(slots, (64 * n + lane) / kPer, 64) * v_tok + kv * a.v_dim + lane % kPer * 8;
                vr[n] = scored_load16(src, lane % kPer * 8 < vreal);
            }
        }
    };
    auto fetch_v = [&](int slots) {
        if constexpr (SAME) stage_from(a.v, slots, v_tok, a.v_dim, v_kv0, vreal, vr);
        else own_v(kv_of(own0), slots);
    };
    auto put_v = [&]() {
        if constexpr (SAME) {
            stage_to(v_all, L::vTile, L::vRow(my_row), vr);
        } else {
#pragma unroll
            for (int n = 0; n < NV; ++n) *reinterpret_cast<scored_u4 *>(v_s + L::vRow((64 * n + lane) / kPer) + lane % kPer * 8) = vr[n];
        }
    };
    // keys by key lane % 32, where they go straight to operands beside values staged by all
    auto near_id = [&](int k0) { return SAME && !L::keys ? talk_block_id(a, table, min(k0 + (lane & 31), end - 1)) : 0; };
    auto near_slot = [&](int id, int k0, int slots) {
        return SAME && !L::keys ? max(talk_slot_of(a, id, min(k0 + (lane & 31), end - 1), end), 0) : slots;
    };
    // 16-byte pieces of a pair's row and of a (head, row)'s keys at places that spread over the banks; inside a piece the place
    // of a wave's weights also turns with key / 4, and that of its keys with head / 4
    auto pair_at = [&](int key, int piece) {
        const int at = HP == 32 ? piece ^ ((l16 >> 1) & 7) : piece ^ ((l16 >> 2) & 3);
        return tm_lds + (key * kTmRows + l16) * L::pair + 16 * at;
    };
    auto weights_at = [&](int head, int piece) { return w_s + (head * kTmRows + l16) * (kTmKeys * 2) + 16 * (piece ^ ((l16 >> 2) & 3)); };

    int slots = slot_of(id_of(0), 0), id = id_of(kTmKeys), id_near = near_id(kTmKeys);
    fetch_k(slots, near_slot(near_id(0), 0, slots));
    fetch_v(slots);
    if constexpr (L::keys) {
        stage_to(k_s, L::kTile, my_row * L::kPitch, kr);
        __syncthreads();
    }
    for (int k0 = 0; k0 < end; k0 += kTmKeys) {
        // ---- scores and weights of keys 16 kb + 4 g + j of row l16 ----
        // (distances first_pos + r - k of 16 rows and 32 keys, from their smallest; a key behind its row gets no weight)
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            const float x = talk_masked_bias(size[i], rate[i], first_pos - (k0 + 31) + lane);
            if (lane < 48) biases[i * 48 + lane] = x;
        }
        tp_own_lds();
        auto weights = [&](int i, int kb, f4 s, float *w) {
            const float *bp = biases + i * 48 + l16 + 31 - 16 * kb - 4 * g;
#pragma unroll
            for (int j = 0; j < 4; ++j) w[j] = __builtin_amdgcn_exp2f(fmaf(s[j], plain, bp[-j]) - (HW == 2 ? 0.f : lse[i]));
        };
        auto put = [&](int kb, float (*w)[4]) {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int key = 16 * kb + 4 * g + j;
                if constexpr (HW == 4) {
                    uint2 hi, lo;
                    la_split2(w[0][j], w[1][j], hi.x, lo.x);
                    la_split2(w[2][j], w[3][j], hi.y, lo.y);
                    *reinterpret_cast<uint2 *>(pair_at(key, wave >> 1) + 8 * ((wave ^ g) & 1)) = hi;
                    *reinterpret_cast<uint2 *>(pair_at(key, 4 + (wave >> 1)) + 8 * ((wave ^ g) & 1)) = lo;
                } else {
                    uint32_t hi, lo;
                    la_split2(w[0][j], w[1][j], hi, lo);
                    *reinterpret_cast<uint32_t *>(pair_at(key, wave >> 2) + 4 * ((wave & 3) ^ g)) = hi;
                    *reinterpret_cast<uint32_t *>(pair_at(key, 2 + (wave >> 2)) + 4 * ((wave & 3) ^ g)) = lo;
                }
            }
        };
        if constexpr (SAME) {
#pragma unroll
            for (int kb = 0; kb < 2; ++kb) {
                float w[HW][4];
                f4 s[HW];
#pragma unroll
                for (int i = 0; i < HW; ++i) s[i] = start[i];
#pragma unroll
                for (int k = 0; k < KS; ++k) {
                    bf8 key;
                    if constexpr (L::keys) key = la_read8(k_s + kv_of(head0) * L::kTile + (16 * kb + l16) * L::kPitch + 32 * k + 8 * g);
                    else key = __builtin_bit_cast(bf8, kr[kb * KS + k]);
#pragma unroll
                    for (int i = 0; i < HW; ++i) s[i] = la_mfma(key, q[i][k], s[i]);
                }
#pragma unroll
                for (int i = 0; i < HW; ++i) weights(i, kb, s[i], w[i]);
                put(kb, w);
                if (HW == 4) __builtin_amdgcn_sched_barrier(0);
            }
        } else {
            float w[2][HW][4];
            int kv = kv_of(head0);
#pragma unroll
            for (int i = 0; i < HW; ++i) {
                if (kv_of(head0 + i) != kv) direct_k(kv = kv_of(head0 + i), slots);
#pragma unroll
                for (int kb = 0; kb < 2; ++kb) {
                    f4 s = start[i];
#pragma unroll
                    for (int k = 0; k < KS; ++k) s = la_mfma(__builtin_bit_cast(bf8, kr[kb * KS + k]), q[i][k], s);
                    weights(i, kb, s, w[kb][i]);
                }
            }
            put(0, w[0]);
            put(1, w[1]);
        }
        const int now = slots;
        // (always, so that waits can be counted: past the last key these are the last key's again)
        slots = slot_of(id, k0 + kTmKeys);
        id = id_of(k0 + 2 * kTmKeys);
        const int near = near_slot(id_near, k0 + kTmKeys, slots);
        id_near = near_id(k0 + 2 * kTmKeys);
        fetch_k(slots, near);
        __builtin_amdgcn_sched_barrier(0);
        __syncthreads();
        // ---- mixed: keys 4 wave .. 4 wave + 3 of row l16, out heads 4 g + i ----
        {
            f4 x[4];
            bf8 one[4];
#pragma unroll
            for (int k = 0; k < 4; ++k) one[k] = la_read8(reinterpret_cast<const __bf16 *>(pair_at(4 * wave + k, g)));
#pragma unroll
            for (int k = 0; k < 4; ++k) x[k] = la_mfma(t_hi, one[k], f4{0.f, 0.f, 0.f, 0.f});
            if (t_rest) {
#pragma unroll
                for (int k = 0; k < 4; ++k) x[k] = la_mfma(t_lo, one[k], x[k]);
            }
            if constexpr (HP == 32) {
#pragma unroll
                for (int k = 0; k < 4; ++k) one[k] = la_read8(reinterpret_cast<const __bf16 *>(pair_at(4 * wave + k, 4 + g)));
#pragma unroll
                for (int k = 0; k < 4; ++k) x[k] = la_mfma(t_hi, one[k], x[k]);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
                *reinterpret_cast<uint2 *>(weights_at(4 * g + i, wave >> 1) + 8 * ((wave ^ g) & 1)) =
                    make_uint2(row_pack_bf16(x[0][i], x[1][i]), row_pack_bf16(x[2][i], x[3][i]));
        }
        put_v();
        if constexpr (L::keys) stage_to(k_s, L::kTile, my_row * L::kPitch, kr);
        fetch_v(slots);
        __builtin_amdgcn_sched_barrier(0);
        __syncthreads();
        // ---- values ----
        bf8 x[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) x[i] = la_read8(reinterpret_cast<const __bf16 *>(weights_at(2 * wave + i, g)));
        const int turn = (wave >> 1 & 1) * 4 * L::vPitch;  // (which four keys come first)
        auto values = [&](int t) {
            const __bf16 *va = v_s + L::vRow(8 * g + (l16 >> 2)) + 16 * t + 4 * (l16 & 3);
            return la_join(la_read_tr(va + turn), la_read_tr(va + 4 * L::vPitch - turn));
        };
        if (SAME || kv_of(own0 + 1) == kv_of(own0)) {
#pragma unroll
            for (int t = 0; t < ET; ++t) {
                const bf8 v = values(t);
#pragma unroll
                for (int i = 0; i < 2; ++i) o[i][t] = la_mfma(v, x[i], o[i][t]);
            }
        } else {
#pragma unroll
            for (int t = 0; t < ET; ++t) o[0][t] = la_mfma(values(t), x[0], o[0][t]);
            own_v(kv_of(own0 + 1), now);
            tp_own_lds();
            put_v();
            tp_own_lds();
#pragma unroll
            for (int t = 0; t < ET; ++t) o[1][t] = la_mfma(values(t), x[1], o[1][t]);
            own_v(kv_of(own0), slots);
        }
        __builtin_amdgcn_sched_barrier(0);
    }
    if (row >= p.n) return;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        if (own0 + i >= a.heads) continue;
        pa_bf16 *out = reinterpret_cast<pa_bf16 *>(a.out) + ((p.row0 + row) * a.heads + own0 + i) * a.vdim;
#pragma unroll
        for (int t = 0; t < ET; ++t) {
            const f4 x = o[i][t];
            const int d = 16 * t + 4 * g;
            if (d >= a.vdim) continue;
            if (FULL || a.vdim % 4 == 0) {
                *reinterpret_cast<uint2 *>(out + d) = make_uint2(row_pack_bf16(x[0], x[1]), row_pack_bf16(x[2], x[3]));
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (d + e < a.vdim) pa_scalar<pa_bf16>::store(out + d + e, x[e]);
            }
        }
    }
}

template <int D, int HW, bool FULL, int NG> int launch_mix(const TalkArgs &a, hipStream_t s) {
    constexpr size_t lds = TmTile<D, HW, NG>::bytes;
    static_assert(lds <= 160 * 1024, "LDS of one compute unit");
    if (int rc = la_big_lds(talk_mix_kernel<D, HW, FULL, NG>, lds, "pa_talking_attention")) return rc;
    const dim3 grid((unsigned)a.batch, (unsigned)((a.max_q_len + kTmRows - 1) / kTmRows), (unsigned)((a.heads + kTmOut - 1) / kTmOut));
    talk_mix_kernel<D, HW, FULL, NG><<<grid, dim3(kTmThreads), lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_talking_attention (portions)");
    return PA_OK;
}
template <int D, int HW> int launch_mix_size(const TalkArgs &a, hipStream_t s) {
    // kv heads beside each other that 16 out heads use at most (all of them, with two heads per wave)
    const int use = HW == 2 ? a.hkv : a.n_rep % kTmOut == 0 ? 1 : kTmOut % a.n_rep == 0 ? kTmOut / a.n_rep : (kTmOut - 2) / a.n_rep + 2;
    if (a.n_rep % HW != 0 || use > 4) return launch_mix<D, HW, false, 0>(a, s);
    return a.n1 == D && a.vdim == D ? launch_mix<D, HW, true, 4>(a, s) : launch_mix<D, HW, false, 4>(a, s);
}

}  // namespace

bool pa_talking_prefill_launch(const TalkArgs &a, int dtype, hipStream_t s, int &rc) {
    const int most = a.n1 > a.vdim ? a.n1 : a.vdim;
    const uintptr_t at = (uintptr_t)a.q1 | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)a.out;
    if (dtype != PA_BF16 || !a.q_lens || most > 128 || a.heads > 32 || (at & 15u) != 0 || a.n1 % 8 != 0 || a.k_dim % 8 != 0 ||
        a.v_dim % 8 != 0 || a.q1_row % 8 != 0 || a.q1_head % 8 != 0 || a.num_blocks * a.bs >= 0x7fffffff || a.bt_stride == 0 || !(a.scale > 0.f))
        return false;
    rc = [&]() -> int {
        const int groups = ((a.max_q_len + 31) / 32 * a.n_rep + 3) / 4;
        PA_REQUIRE(groups <= 65535, "pa_talking_attention: max_q_len=%d is too long for one launch", a.max_q_len);
        const dim3 grid((unsigned)a.batch, (unsigned)a.hkv, (unsigned)groups);
        if (a.n1 <= 64) talk_sums_kernel<64><<<grid, dim3(256), 0, s>>>(a);
        else talk_sums_kernel<128><<<grid, dim3(256), 0, s>>>(a);
        PA_CHECK_LAUNCH("pa_talking_attention (sums)");
        if (a.heads <= 16) return most <= 64 ? launch_mix_size<64, 2>(a, s) : launch_mix_size<128, 2>(a, s);
        return most <= 64 ? launch_mix_size<64, 4>(a, s) : launch_mix_size<128, 4>(a, s);
    }();
    return true;
}
