// Decode steps of attention with score terms on the matrix cores (16-bit pools): one row per sequence, a workgroup per
// (kv head, 16 QT of its query heads, piece of the sequence's keys).
//
// A tile of 64 keys goes from memory through registers into LDS while the tile before it is multiplied.  Each of four
// waves scores 16 of its keys for all query heads (S^T = K Q^T; with eight waves, for half of them), the probabilities go
// through LDS, then each wave multiplies all 64 keys into its share of the value columns (O^T += V^T P^T, V^T by transposing
// LDS reads).  With one tensor for keys
// and values (latent attention) the tile is read from memory once for both.
#include "scored_attn.h"

namespace {

typedef __bf16 sd_bf8 __attribute__((ext_vector_type(8)));
typedef float sd_f4 __attribute__((ext_vector_type(4)));
typedef short sd_s4 __attribute__((ext_vector_type(4)));

constexpr int kSdKeys = 64;

__device__ __forceinline__ sd_f4 sd_mfma(sd_bf8 x, sd_bf8 y, sd_f4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, y, c, 0, 0, 0); }
__device__ __forceinline__ sd_bf8 sd_read8(const __bf16 *p) { return *reinterpret_cast<const sd_bf8 *>(p); }
// Lane i of 16: elements (4 keys, column i) of the 4 x 16 block whose lane s holds key s / 4, columns 4 (s % 4) ..
__device__ __forceinline__ sd_s4 sd_tr(const __bf16 *p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((sd_s4 __attribute__((address_space(3))) *)p);
}

// KC, VC: key and value elements held (multiples of 32 and 64).  ONE: values are the keys' first columns.  A workgroup whose
// tile fills the LDS of a compute unit has eight waves where its queries fill them.
template <int KC, int VC, bool ONE, int QT> struct SdTile {
    static constexpr int waves = KC >= 512 && QT > 1 ? 8 : 4, threads = 64 * waves;
    static constexpr int kPitch = KC + 8, vPitch = ONE ? KC + 8 : VC + 8;
    static constexpr int kElems = kSdKeys * kPitch, vElems = ONE ? 0 : kSdKeys * vPitch, qElems = 16 * QT * kPitch;
    static constexpr int pPitch = kSdKeys + 8, pElems = 16 * QT * pPitch;
    static constexpr size_t bytes = (size_t)(kElems + vElems + qElems + pElems) * 2 + 4 * 16 * QT * 4;
};

template <int KC, int VC, bool ONE, int QT>
__global__ __launch_bounds__((SdTile<KC, VC, ONE, QT>::threads)) void scored_decode_kernel(const ScoredArgs a) {
    using L = SdTile<KC, VC, ONE, QT>;
    constexpr int kThr = L::threads, kVT = VC / 16 / L::waves;       // value column tiles per wave
    constexpr int kTQ = QT * 4 / L::waves;                           // query tiles that a wave scores
    constexpr int kKL = kSdKeys * KC / 8 / kThr, kVL = ONE ? 0 : kSdKeys * VC / 8 / kThr;  // 16-byte loads per thread and tile
    static_assert(kSdKeys * KC / 8 % kThr == 0 && VC % (16 * L::waves) == 0 && kTQ > 0, "whole loads");
    extern __shared__ __align__(16) char sd_lds[];
    __bf16 *ks = reinterpret_cast<__bf16 *>(sd_lds), *vs = ONE ? ks : ks + L::kElems;
    __bf16 *qs = ks + L::kElems + L::vElems, *ps = qs + L::qElems;
    float *tops = reinterpret_cast<float *>(ps + L::pElems);  // [4 key groups][16 QT]
    const int groups = (a.n_rep + 16 * QT - 1) / (16 * QT);
    const int kvh = blockIdx.x / groups, rep0 = blockIdx.x % groups * 16 * QT, piece = blockIdx.y, b = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const int kg = wave & 3, t0 = wave / 4 * kTQ;  // the wave's keys of a tile, its first query tile
    const int pos = a.ctx_lens[b] - 1, h0 = kvh * a.n_rep + rep0, n_heads = min(16 * QT, a.n_rep - rep0);
    if (pos < 0) return;  // padding
    const int first = scored_first_key(a, pos), per = ((pos + 1 - first + a.splits - 1) / a.splits + kSdKeys - 1) / kSdKeys * kSdKeys;
    const int lo = first + piece * per, end = min(pos + 1, lo + per);
    float *ml = a.part_ml + ((int64_t)b * a.heads + h0) * a.splits * 2 + piece * 2;
    if (lo >= end) {
        if (a.splits > 1 && tid < n_heads) ml[tid * a.splits * 2 + 1] = 0.f;
        return;
    }
    // ---- queries ----
    const uint16_t *q1 = reinterpret_cast<const uint16_t *>(a.q1) + b * a.q1_row, *q2 = reinterpret_cast<const uint16_t *>(a.q2) + b * a.q2_row;
    uint16_t *qw = reinterpret_cast<uint16_t *>(qs);
    for (int i = tid; i < 16 * QT * (KC / 8); i += kThr) {
        const int r = i / (KC / 8), e = i % (KC / 8) * 8;
        uint4 x = make_uint4(0, 0, 0, 0);
        if (r < n_heads) {
            if (e + 8 <= a.n1) x = *reinterpret_cast<const uint4 *>(q1 + (h0 + r) * a.q1_head + e);
            else if (e >= a.n1 && e + 8 <= a.n1 + a.n2) x = *reinterpret_cast<const uint4 *>(q2 + (h0 + r) * a.q2_head + (e - a.n1));
        }
        *reinterpret_cast<uint4 *>(qw + r * L::kPitch + e) = x;
    }
    // ---- tiles ----
    const int32_t *table = a.bt + b * a.bt_stride;
    const int kreal = (a.n1 + a.n2 + 7) / 8 * 8, vreal = (a.vdim + 7) / 8 * 8;
    const uint16_t *kp = reinterpret_cast<const uint16_t *>(a.k) + (int64_t)kvh * a.k_dim, *vp = reinterpret_cast<const uint16_t *>(a.v) + (int64_t)kvh * a.v_dim;
    const int64_t k_tok = (int64_t)a.hkv * a.k_dim, v_tok = (int64_t)a.hkv * a.v_dim;
    auto id_of = [&](int k0) { return scored_block_id(a, table, min(k0 + lane, end - 1)); };
    scored_u4 kr[kKL], vr[kVL ? kVL : 1];
    auto fetch = [&](int id, int k0) {
        const int slots = scored_slot_of(a, id, k0 + lane, end);
#pragma unroll
        for (int n = 0; n < kKL; ++n) {
            const int c = tid + kThr * n, s = __shfl(slots, c / (KC / 8), 64), e = c % (KC / 8) * 8;
            kr[n] = scored_load16(kp + s * k_tok + e, s >= 0 && e < kreal);
        }
        if constexpr (!ONE) {
#pragma unroll
            for (int n = 0; n < kVL; ++n) {
                const int c = tid + kThr * n, s = __shfl(slots, c / (VC / 8), 64), e = c % (VC / 8) * 8;
                vr[n] = scored_load16(vp + s * v_tok + e, s >= 0 && e < vreal);
            }
        }
    };
    sd_f4 o[QT][kVT];
    float m[QT], l[kTQ];
#pragma unroll
    for (int t = 0; t < kTQ; ++t) l[t] = 0.f;
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        m[t] = kScoredNone;
#pragma unroll
        for (int c = 0; c < kVT; ++c) o[t][c] = sd_f4{0.f, 0.f, 0.f, 0.f};
    }
    const float to2 = kScoredLog2e, plain = a.scale * kScoredLog2e, cap_in = a.cap > 0.f ? 2.f * plain / a.cap : 0.f  /* tanh(z) = 1 - 2 / (1 + e^(2z)) */, cap_out = a.cap * kScoredLog2e;
    const float *bias[kTQ];  // of this lane's heads
#pragma unroll
    for (int t = 0; t < kTQ; ++t) bias[t] = a.bias + (int64_t)(h0 + min(16 * (t0 + t) + l16, n_heads - 1)) * a.bias_n;
    fetch(id_of(lo), lo);
    int id = id_of(lo + kSdKeys);
    for (int k0 = lo; k0 < end; k0 += kSdKeys) {
#pragma unroll
        for (int n = 0; n < kKL; ++n) {
            const int c = tid + kThr * n;
            *reinterpret_cast<scored_u4 *>(ks + c / (KC / 8) * L::kPitch + c % (KC / 8) * 8) = kr[n];
        }
        if constexpr (!ONE) {
#pragma unroll
            for (int n = 0; n < kVL; ++n) {
                const int c = tid + kThr * n;
                *reinterpret_cast<scored_u4 *>(vs + c / (VC / 8) * L::vPitch + c % (VC / 8) * 8) = vr[n];
            }
        }
        __syncthreads();
        const int key = k0 + 16 * kg + 4 * g;
        float near[kTQ][4];  // biases: ahead of the next tile's loads, which they do not wait for
        if (a.bias) {
#pragma unroll
            for (int t = 0; t < kTQ; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) near[t][i] = bias[t][min(max(pos - key - i, 0), a.bias_n - 1)];
        }
        if (k0 + kSdKeys < end) {
            fetch(id, k0 + kSdKeys);
            id = id_of(k0 + 2 * kSdKeys);
        }
        // scores: keys k0 + 16 wave + 4 g + i, head l16 of its query tiles
        sd_f4 s[kTQ];
#pragma unroll
        for (int t = 0; t < kTQ; ++t) s[t] = sd_f4{0.f, 0.f, 0.f, 0.f};
        const __bf16 *ka = ks + (16 * kg + l16) * L::kPitch + 8 * g, *qa = qs + (16 * t0 + l16) * L::kPitch + 8 * g;
#pragma unroll
        for (int kk = 0; kk < KC / 32; ++kk) {
            const sd_bf8 x = sd_read8(ka + 32 * kk);
#pragma unroll
            for (int t = 0; t < kTQ; ++t) s[t] = sd_mfma(x, sd_read8(qa + 16 * t * L::kPitch + 32 * kk), s[t]);
        }
        if (a.cap > 0.f) {  // (in units of the base-2 exponential)
#pragma unroll
            for (int t = 0; t < kTQ; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) s[t][i] = cap_out - 2.f * cap_out * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s[t][i] * cap_in));
        } else {
#pragma unroll
            for (int t = 0; t < kTQ; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) s[t][i] *= plain;
        }
        if (a.bias) {
#pragma unroll
            for (int t = 0; t < kTQ; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) s[t][i] = fmaf(near[t][i], to2, s[t][i]);
        }
#pragma unroll
        for (int t = 0; t < kTQ; ++t) {
            const int r = 16 * (t0 + t) + l16;
            float top = kScoredNone;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                s[t][i] = key + i < end ? s[t][i] : kScoredNone;
                top = fmaxf(top, s[t][i]);
            }
            top = fmaxf(top, __shfl_xor(top, 16, 64));
            top = fmaxf(top, __shfl_xor(top, 32, 64));
            if (g == 0) tops[kg * 16 * QT + r] = top;
        }
        __syncthreads();
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            const int r = 16 * t + l16;
            float next = m[t];
#pragma unroll
            for (int w = 0; w < 4; ++w) next = fmaxf(next, tops[w * 16 * QT + r]);
            const float keep = __builtin_amdgcn_exp2f(m[t] - next);
            m[t] = next;
            if (kTQ == QT || t / kTQ == wave / 4) {
                const int own = t % kTQ;
                float p[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) p[i] = __builtin_amdgcn_exp2f(s[own][i] - next);
                l[own] = fmaf(l[own], keep, (p[0] + p[1]) + (p[2] + p[3]));
                *reinterpret_cast<uint2 *>(ps + r * L::pPitch + 16 * kg + 4 * g) = make_uint2(row_pack_bf16(p[0], p[1]), row_pack_bf16(p[2], p[3]));
            }
#pragma unroll
            for (int c = 0; c < kVT; ++c)
#pragma unroll
                for (int i = 0; i < 4; ++i) o[t][c][i] *= keep;
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            sd_bf8 p[QT];
#pragma unroll
            for (int t = 0; t < QT; ++t) p[t] = sd_read8(ps + (16 * t + l16) * L::pPitch + 32 * kk + 8 * g);
#pragma unroll
            for (int c = 0; c < kVT; ++c) {
                const __bf16 *va = vs + (32 * kk + 8 * g + (l16 >> 2)) * L::vPitch + 16 * (wave * kVT + c) + 4 * (l16 & 3);
                const sd_s4 x = sd_tr(va), y = sd_tr(va + 4 * L::vPitch);
                typedef short s8 __attribute__((ext_vector_type(8)));
                const sd_bf8 v8 = __builtin_bit_cast(sd_bf8, s8{x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]});
#pragma unroll
                for (int t = 0; t < QT; ++t) o[t][c] = sd_mfma(v8, p[t], o[t][c]);
            }
        }
        __syncthreads();
    }
    // ---- sums over the waves, then out ----
#pragma unroll
    for (int t = 0; t < kTQ; ++t) {
        l[t] += __shfl_xor(l[t], 16, 64);
        l[t] += __shfl_xor(l[t], 32, 64);
        if (g == 0) tops[kg * 16 * QT + 16 * (t0 + t) + l16] = l[t];
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int r = 16 * t + l16;
        if (r >= n_heads) continue;
        float sum = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) sum += tops[w * 16 * QT + r];
        if (a.splits > 1) {
            if (wave == 0 && g == 0) {
                ml[r * a.splits * 2] = m[t];
                ml[r * a.splits * 2 + 1] = sum;
            }
            float *dst = a.part_o + (((int64_t)b * a.heads + h0 + r) * a.splits + piece) * VC;
#pragma unroll
            for (int c = 0; c < kVT; ++c) *reinterpret_cast<sd_f4 *>(dst + 16 * (wave * kVT + c) + 4 * g) = o[t][c];
            continue;
        }
        float keep = 1.f;
        if (a.sink) {
            const float sink = a.sink[h0 + r] * to2, all = fmaxf(m[t], sink);
            keep = __builtin_amdgcn_exp2f(m[t] - all);
            sum = fmaf(sum, keep, __builtin_amdgcn_exp2f(sink - all));
        }
        const float f = keep / sum;
        pa_bf16 *dst = reinterpret_cast<pa_bf16 *>(a.out) + ((int64_t)b * a.heads + h0 + r) * a.vdim;
#pragma unroll
        for (int c = 0; c < kVT; ++c) {
            const int d = 16 * (wave * kVT + c) + 4 * g;
            if (d >= a.vdim) continue;
            if (a.vdim % 4 == 0) {
                *reinterpret_cast<uint2 *>(dst + d) = make_uint2(row_pack_bf16(o[t][c][0] * f, o[t][c][1] * f), row_pack_bf16(o[t][c][2] * f, o[t][c][3] * f));
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (d + i < a.vdim) pa_scalar<pa_bf16>::store(dst + d + i, o[t][c][i] * f);
            }
        }
    }
}

// Pieces of a sequence's keys joined: a wave per (row, head), four value columns per lane and turn
__global__ __launch_bounds__(64) void scored_merge_kernel(const ScoredArgs a, int vc) {
    const int64_t rh = blockIdx.x;
    const int h = (int)(rh % a.heads);
    if (a.ctx_lens[rh / a.heads] < 1) return;
    const float *ml = a.part_ml + rh * a.splits * 2;
    float m = a.sink ? a.sink[h] * kScoredLog2e : kScoredNone;
    for (int s = 0; s < a.splits; ++s)
        if (ml[2 * s + 1] > 0.f) m = fmaxf(m, ml[2 * s]);
    for (int d = threadIdx.x * 4; d < a.vdim; d += 256) {
        const float *po = a.part_o + rh * a.splits * vc + d;
        float den = a.sink ? __builtin_amdgcn_exp2f(a.sink[h] * kScoredLog2e - m) : 0.f;
        sd_f4 num = sd_f4{0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < a.splits; ++s) {
            if (!(ml[2 * s + 1] > 0.f)) continue;  // (a piece without keys wrote no values)
            const float w = __builtin_amdgcn_exp2f(ml[2 * s] - m);
            const sd_f4 x = *reinterpret_cast<const sd_f4 *>(po + (int64_t)s * vc);
            den = fmaf(w, ml[2 * s + 1], den);
#pragma unroll
            for (int i = 0; i < 4; ++i) num[i] = fmaf(w, x[i], num[i]);
        }
        pa_bf16 *out = reinterpret_cast<pa_bf16 *>(a.out) + rh * a.vdim + d;
        const float f = 1.f / den;
        if (a.vdim % 4 == 0) {
            *reinterpret_cast<uint2 *>(out) = make_uint2(row_pack_bf16(num[0] * f, num[1] * f), row_pack_bf16(num[2] * f, num[3] * f));
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (d + i < a.vdim) pa_scalar<pa_bf16>::store(out + i, num[i] * f);
        }
    }
}

template <int KC, int VC, bool ONE, int QT> int launch_decode(const ScoredArgs &a, hipStream_t s) {
    constexpr size_t lds = SdTile<KC, VC, ONE, QT>::bytes;
    static_assert(lds <= 160 * 1024, "LDS of one compute unit");
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(scored_decode_kernel<KC, VC, ONE, QT>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return pa_fail(PA_ERR_HIP, "pa_scored_attention: %s", hipGetErrorString(e));
    }
    const int groups = (a.n_rep + 16 * QT - 1) / (16 * QT);
    scored_decode_kernel<KC, VC, ONE, QT><<<dim3((unsigned)(a.hkv * groups), (unsigned)a.splits, (unsigned)a.batch), dim3(SdTile<KC, VC, ONE, QT>::threads), lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_scored_attention (decode)");
    if (a.splits > 1) {
        scored_merge_kernel<<<dim3((unsigned)(a.batch * a.heads)), dim3(64), 0, s>>>(a, VC);
        PA_CHECK_LAUNCH("pa_scored_attention (merge)");
    }
    return PA_OK;
}

template <int KC, int VC> int launch_one(const ScoredArgs &a, hipStream_t s) {
    if (a.n_rep <= 16) return launch_decode<KC, VC, true, 1>(a, s);
    if (a.n_rep <= 32) return launch_decode<KC, VC, true, 2>(a, s);
    return launch_decode<KC, VC, true, 4>(a, s);
}

}  // namespace

bool pa_scored_decode_launch(const ScoredArgs &a, int dtype, hipStream_t s, int &rc) {
    const int keys = a.n1 + a.n2, vc = scored_value_cols(keys, a.vdim, a.v == a.k);
    const uintptr_t at = (uintptr_t)a.q1 | (uintptr_t)a.q2 | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)a.out;
    if (dtype != PA_BF16 || a.q_lens || vc == 0 || (at & 15u) != 0 || a.n1 % 8 != 0 || a.n2 % 8 != 0 || a.k_dim % 8 != 0 ||
        a.v_dim % 8 != 0 || a.q1_row % 8 != 0 || a.q1_head % 8 != 0 || a.q2_row % 8 != 0 || a.q2_head % 8 != 0 ||
        a.num_blocks * a.bs >= 0x7fffffff || a.bt_stride == 0 || !(a.scale > 0.f))
        return false;
    if (a.v == a.k) rc = vc == 128 ? launch_one<160, 128>(a, s) : vc == 256 ? launch_one<320, 256>(a, s) : launch_one<576, 512>(a, s);
    else rc = vc == 64 ? launch_decode<64, 64, false, 1>(a, s) : vc == 128 ? launch_decode<128, 128, false, 1>(a, s) : launch_decode<256, 256, false, 1>(a, s);
    return true;
}
