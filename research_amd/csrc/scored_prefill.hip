// Portions of prompts of attention with score terms on the matrix cores (16-bit pools, keys and values of up to 256).
//
// A wave owns 32 rows of one query head, a workgroup four (row block, head) pairs of one kv head in turn, which share tiles of
// 64 keys and values in LDS; the next tile is on its way in registers.  As in prefill_mfma.h everything is transposed:
// S^T = K Q^T leaves a lane 16 keys of one row, which in register order are the operand of O^T += V^T P^T.  The distance
// biases of a wave's head lie in LDS, newest key last, with margins on both sides, so that a lane reads the biases of
// consecutive keys side by side and nothing is clamped; blocks of keys past the last distance share one number.
#include "prefill_mfma.h"
#include "scored_attn.h"

namespace {

using namespace pa_decode_detail;

constexpr int kSpKeys = 64, kSpMargin = 64, kSpMaxBias = 4096;
constexpr float kSpSlack = 8.f;  // log2 of the factor by which a row's reference maximum may lag

template <int DK, int DV> struct SpTile {
    static constexpr int k_pitch = DK + 8, v_pitch = DV + 8;
    static constexpr size_t tiles = (size_t)kSpKeys * (k_pitch + v_pitch) * 2;
};

template <int DK, int DV, bool CAP> __global__ __launch_bounds__(256, DV == 256 ? 1 : 2) void scored_prefill_kernel(const ScoredArgs a, int bias_n) {
    using M = Mfma16<pa_bf16>;
    using X8 = M::x8;
    using X4 = M::x4;
    using L = SpTile<DK, DV>;
    constexpr int KS = DK / 16, DT = DV / 32, NK = kSpKeys * DK / 8 / 256, NV = kSpKeys * DV / 8 / 256;
    extern __shared__ __align__(16) char sp_lds[];
    uint16_t *ks = reinterpret_cast<uint16_t *>(sp_lds), *vs = ks + kSpKeys * L::k_pitch;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), half = lane >> 5, col = lane & 31;
    const int table_n = bias_n + 2 * kSpMargin;
    float *bias = reinterpret_cast<float *>(sp_lds + L::tiles) + wave * table_n;
    const int kvh = blockIdx.x, b = blockIdx.z;
    ScoredPortion p;
    if (!scored_portion(a, b, p)) return;
    const int n_tasks = (p.n + 31) / 32 * a.n_rep;
    const int group = gridDim.y - 1 - blockIdx.y;  // (the rows with the most keys first)
    if (group * 4 >= n_tasks) return;
    const int task = group * 4 + wave, last_task = min(n_tasks, group * 4 + 4) - 1;
    const bool live = task < n_tasks;
    const int row0 = (live ? task / a.n_rep : 0) * 32, h = kvh * a.n_rep + (live ? task % a.n_rep : 0);
    const int row = row0 + col, pos = p.pos0 + min(row, p.n - 1);
    const int my_first = scored_first_key(a, pos);                       // this lane's row: first key, last key is pos
    const int wave_lo = scored_first_key(a, p.pos0 + row0), wave_hi = p.pos0 + min(row0 + 32, p.n);  // keys [lo, hi) of the wave
    const int wg_lo = scored_first_key(a, p.pos0 + group * 4 / a.n_rep * 32);
    const int wg_hi = p.pos0 + min(last_task / a.n_rep * 32 + 32, p.n);
    const float to2 = kScoredLog2e, plain = a.scale * kScoredLog2e;
    const float cap_in = CAP ? 2.f * plain / a.cap : 0.f, cap_out = a.cap * kScoredLog2e;  // tanh(z) = 1 - 2 / (1 + e^(2z))
    // bias[kSpMargin - 1 + bias_n - dist]: one entry per distance from bias_n - 1 + kSpMargin down to -kSpMargin
    const float shift = CAP ? cap_out : 0.f;
    for (int i = lane; i < table_n; i += 64) {
        const int dist = min(max(kSpMargin - 1 + bias_n - i, 0), bias_n - 1);
        bias[i] = (a.bias ? a.bias[(int64_t)h * a.bias_n + dist] * to2 : 0.f) + shift;
    }
    const float far = (a.bias ? a.bias[(int64_t)h * a.bias_n + bias_n - 1] * to2 : 0.f) + shift;
    X8 q[KS];
    {
        const uint16_t *src = reinterpret_cast<const uint16_t *>(a.q1) + (p.row0 + min(row, p.n - 1)) * a.q1_row + h * a.q1_head;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int d = 16 * k + 8 * half;
            q[k] = __builtin_bit_cast(X8, d < a.n1 ? *reinterpret_cast<const uint4 *>(src + d) : make_uint4(0, 0, 0, 0));
        }
    }
    f32x16 o[DT];
#pragma unroll
    for (int t = 0; t < DT; ++t)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[t][i] = 0.f;
    float m = a.sink ? a.sink[h] * to2 : kScoredNone, l = a.sink && half == 0 ? 1.f : 0.f;

    const int32_t *table = a.bt + b * a.bt_stride;
    const uint16_t *kp = reinterpret_cast<const uint16_t *>(a.k) + (int64_t)kvh * a.k_dim, *vp = reinterpret_cast<const uint16_t *>(a.v) + (int64_t)kvh * a.v_dim;
    const int64_t k_tok = (int64_t)a.hkv * a.k_dim, v_tok = (int64_t)a.hkv * a.v_dim;
    const int kreal = (a.n1 + 7) / 8 * 8, vreal = (a.vdim + 7) / 8 * 8;
    auto id_of = [&](int k0) { return scored_block_id(a, table, min(k0 + lane, wg_hi - 1)); };
    scored_u4 kr[NK], vr[NV];
    auto fetch = [&](int id, int k0) {
        const int slots = scored_slot_of(a, id, k0 + lane, wg_hi);
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            const int c = tid + 256 * n, s = __shfl(slots, c / (DK / 8), 64), e = c % (DK / 8) * 8;
            kr[n] = scored_load16(kp + s * k_tok + e, s >= 0 && e < kreal);
        }
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const int c = tid + 256 * n, s = __shfl(slots, c / (DV / 8), 64), e = c % (DV / 8) * 8;
            vr[n] = scored_load16(vp + s * v_tok + e, s >= 0 && e < vreal);
        }
    };
    const int g16 = lane >> 4, s16 = lane & 15;
    const uint16_t *v_at = vs + (4 * (g16 >> 1) + (s16 >> 2)) * L::v_pitch + 16 * (g16 & 1) + 4 * (s16 & 3);
    const int k_start = wg_lo / kSpKeys * kSpKeys;
    fetch(id_of(k_start), k_start);
    int id = id_of(k_start + kSpKeys);
    for (int k0 = k_start; k0 < wg_hi; k0 += kSpKeys) {
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            const int c = tid + 256 * n;
            *reinterpret_cast<scored_u4 *>(ks + c / (DK / 8) * L::k_pitch + c % (DK / 8) * 8) = kr[n];
        }
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const int c = tid + 256 * n;
            *reinterpret_cast<scored_u4 *>(vs + c / (DV / 8) * L::v_pitch + c % (DV / 8) * 8) = vr[n];
        }
        __syncthreads();
        if (k0 + kSpKeys < wg_hi) {
            fetch(id, k0 + kSpKeys);
            id = id_of(k0 + 2 * kSpKeys);
        }
#pragma unroll
        for (int sub = 0; sub < 2; ++sub) {
            const int kb = k0 + 32 * sub;  // (uniform per wave)
            if (!live || kb >= wave_hi || kb + 32 <= wave_lo) continue;
            f32x16 s;
#pragma unroll
            for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
            for (int k = 0; k < KS; ++k)
                s = M::mma(__builtin_bit_cast(X8, *reinterpret_cast<const uint4 *>(ks + (32 * sub + col) * L::k_pitch + 16 * k + 8 * half)), q[k], s);
            // element i: key kb + 8 (i / 4) + 4 half + i % 4
            const bool is_far = p.pos0 + row0 - (kb + 31) >= bias_n - 1;  // every distance shares the last bias
            const float *bp = bias + kSpMargin - 1 + bias_n - (p.pos0 + row) + kb + 4 * half;
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const float add = is_far ? far : bp[8 * (i >> 2) + (i & 3)];
                if constexpr (CAP) s[i] = fmaf(-2.f * cap_out, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s[i] * cap_in)), add);
                else s[i] = fmaf(s[i], plain, add);
            }
            if (kb + 31 > p.pos0 + row0 || kb < scored_first_key(a, wave_hi - 1)) {
                const int hi = pos - kb - 4 * half, lo = my_first - kb - 4 * half;
#pragma unroll
                for (int i = 0; i < 16; ++i) {
                    const int idx = 8 * (i >> 2) + (i & 3);
                    s[i] = idx <= hi && idx >= lo ? s[i] : kScoredNone;
                }
            }
            float top = fmaxf(s[0], s[1]);
#pragma unroll
            for (int i = 2; i < 16; ++i) top = fmaxf(top, s[i]);
            top = fmaxf(top, __shfl_xor(top, 32, 64));
            if (__ballot(top > m + kSpSlack) != 0) {
                const float next = fmaxf(m, top), keep = __builtin_amdgcn_exp2f(m - next);
                m = next;
                l *= keep;
#pragma unroll
                for (int t = 0; t < DT; ++t)
#pragma unroll
                    for (int i = 0; i < 16; ++i) o[t][i] *= keep;
            }
            uint32_t w[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float x = __builtin_amdgcn_exp2f(s[2 * i] - m), y = __builtin_amdgcn_exp2f(s[2 * i + 1] - m);
                l += x + y;
                w[i] = row_pack_bf16(x, y);
            }
#pragma unroll
            for (int k2 = 0; k2 < 2; ++k2) {
                const X8 pb = __builtin_bit_cast(X8, make_uint4(w[4 * k2], w[4 * k2 + 1], w[4 * k2 + 2], w[4 * k2 + 3]));
#pragma unroll
                for (int t = 0; t < DT; ++t) {
                    const uint16_t *at = v_at + (32 * sub + 16 * k2) * L::v_pitch + 32 * t;
                    const X4 x = M::tr_read(at), y = M::tr_read(at + 8 * L::v_pitch);
                    X8 va;
#pragma unroll
                    for (int e = 0; e < 4; ++e) { va[e] = x[e]; va[4 + e] = y[e]; }
                    o[t] = M::mma(va, pb, o[t]);
                }
            }
        }
        __syncthreads();
    }
    const float f = 1.f / (l + __shfl_xor(l, 32, 64));
    if (!live || row >= p.n) return;
    pa_bf16 *out = reinterpret_cast<pa_bf16 *>(a.out) + ((p.row0 + row) * a.heads + h) * a.vdim;
#pragma unroll
    for (int t = 0; t < DT; ++t)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
            const int d = 32 * t + 8 * g + 4 * half;
            if (d >= a.vdim) continue;
            if (a.vdim % 4 == 0) {
                *reinterpret_cast<uint2 *>(out + d) = make_uint2(row_pack_bf16(o[t][4 * g] * f, o[t][4 * g + 1] * f),
                                                                 row_pack_bf16(o[t][4 * g + 2] * f, o[t][4 * g + 3] * f));
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (d + i < a.vdim) pa_scalar<pa_bf16>::store(out + d + i, o[t][4 * g + i] * f);
            }
        }
}

template <int DK, int DV, bool CAP> int launch_prefill(const ScoredArgs &a, int bias_n, hipStream_t s) {
    const size_t lds = SpTile<DK, DV>::tiles + (size_t)4 * (bias_n + 2 * kSpMargin) * sizeof(float);
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(scored_prefill_kernel<DK, DV, CAP>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "pa_scored_attention: %s", hipGetErrorString(e));
    }
    const int groups = ((a.max_q_len + 31) / 32 * a.n_rep + 3) / 4;
    PA_REQUIRE(groups <= 65535, "pa_scored_attention: max_q_len=%d is too long for one launch", a.max_q_len);
    scored_prefill_kernel<DK, DV, CAP><<<dim3((unsigned)a.hkv, (unsigned)groups, (unsigned)a.batch), dim3(256), lds, s>>>(a, bias_n);
    PA_CHECK_LAUNCH("pa_scored_attention (portions)");
    return PA_OK;
}

template <int DK, int DV> int launch_prefill_cap(const ScoredArgs &a, int bias_n, hipStream_t s) {
    return a.cap > 0.f ? launch_prefill<DK, DV, true>(a, bias_n, s) : launch_prefill<DK, DV, false>(a, bias_n, s);
}

}  // namespace

bool pa_scored_prefill_launch(const ScoredArgs &a, int dtype, hipStream_t s, int &rc) {
    const int most = a.n1 > a.vdim ? a.n1 : a.vdim;
    const uintptr_t at = (uintptr_t)a.q1 | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)a.out;
    int bias_n = a.bias ? a.bias_n : 1;
    if (a.window > 0 && bias_n > a.window) bias_n = a.window;  // (no distance reaches the window)
    if (dtype != PA_BF16 || !a.q_lens || a.n2 != 0 || most > 256 || bias_n > kSpMaxBias || (at & 15u) != 0 || a.n1 % 8 != 0 ||
        a.k_dim % 8 != 0 || a.v_dim % 8 != 0 || a.q1_row % 8 != 0 || a.q1_head % 8 != 0 || a.num_blocks * a.bs >= 0x7fffffff ||
        a.bt_stride == 0 || !(a.scale > 0.f))
        return false;
    rc = most <= 64                        ? launch_prefill_cap<64, 64>(a, bias_n, s)
         : most <= 128                     ? launch_prefill_cap<128, 128>(a, bias_n, s)
         : a.n1 <= 192 && a.vdim <= 128    ? launch_prefill_cap<192, 128>(a, bias_n, s)
                                           : launch_prefill_cap<256, 256>(a, bias_n, s);
    return true;
}
