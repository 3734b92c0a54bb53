// Decode steps of attention with mixed heads on the matrix cores (16-bit pools): one row per sequence, a workgroup per (kv head,
// 16 of its query heads, piece of the sequence's keys).
//
// A first kernel reads the keys: scores S^T = K Q^T straight from memory into operands, a wave for 16 keys at a time, kept in
// the workspace (4 bytes per key and head beside a key's 2 dim bytes per kv head), with the piece's largest score and sum.  A
// second one reads the values: it turns the scores of all heads into weights (the sums of all pieces are known by now),
// multiplies them by the mixing matrix and the result into the values, 64 keys at a time; every wave has its value columns and
// mixes for itself (W^T = P^T T^T leaves a lane four keys of one head, which are the operand of O^T += V^T W^T in register
// order).  Pieces just add up, since weights enter normalised.
#include "linear_tiles.h"
#include "talking.h"

namespace {

constexpr int kTdKeys = 64, kTdMaxSplits = 16;

int td_value_cols(int vdim) { return vdim <= 64 ? 64 : vdim <= 128 ? 128 : 256; }

struct TdPiece {
    int lo, end;
};
__device__ __forceinline__ TdPiece td_piece(const TalkArgs &a, int keys, int piece) {
    const int per = ((keys + a.splits - 1) / a.splits + kTdKeys - 1) / kTdKeys * kTdKeys, lo = piece * per;
    return {lo, min(keys, lo + per)};
}

template <int KC> __global__ __launch_bounds__(256) void talk_scores_kernel(const TalkArgs a) {
    __shared__ float ms[4][16], ls[4][16];
    const int groups = (a.n_rep + 15) / 16, kvh = blockIdx.x / groups, rep0 = blockIdx.x % groups * 16, piece = blockIdx.y, b = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const int keys = a.ctx_lens[b], h0 = kvh * a.n_rep + rep0, n_heads = min(16, a.n_rep - rep0);
    if (keys <= 0) return;  // padding
    const TdPiece p = td_piece(a, keys, piece);
    if (p.lo >= p.end) return;
    const int h = h0 + min(l16, n_heads - 1);
    bf8 q[KC / 32];
    {
        const uint16_t *src = reinterpret_cast<const uint16_t *>(a.q1) + b * a.q1_row + h * a.q1_head;
#pragma unroll
        for (int kk = 0; kk < KC / 32; ++kk) q[kk] = __builtin_bit_cast(bf8, scored_load16(src + 32 * kk + 8 * g, 32 * kk + 8 * g < a.n1));
    }
    const float plain = a.scale * kScoredLog2e, size = a.size ? a.size[h] : 0.f, rate = a.rate ? a.rate[h] : 0.f;
    const int32_t *table = a.bt + b * a.bt_stride;
    const uint16_t *kp = reinterpret_cast<const uint16_t *>(a.k) + (int64_t)kvh * a.k_dim + 8 * g;
    const int64_t k_tok = (int64_t)a.hkv * a.k_dim;
    scored_u4 x[2][KC / 32];
    auto fetch = [&](scored_u4 *to, int key) {
        const int slot = talk_slot_of(a, talk_block_id(a, table, min(key, p.end - 1)), key, p.end);
        const uint16_t *src = kp + (int64_t)max(slot, 0) * k_tok;
#pragma unroll
        for (int kk = 0; kk < KC / 32; ++kk) to[kk] = scored_load16(src + 32 * kk, slot >= 0 && 32 * kk + 8 * g < a.n1);
    };
    float m = kScoredNone, l = 0.f;
    float *dst = a.scores + ((int64_t)b * a.heads + h) * a.keys_cap;
    auto tile = [&](const scored_u4 *k, int k0) {  // keys k0 + 4 g + i of head l16
        f4 s = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < KC / 32; ++kk) s = la_mfma(__builtin_bit_cast(bf8, k[kk]), q[kk], s);
        const int key = k0 + 4 * g;
        float top = kScoredNone;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            s[i] *= plain;
            if (a.size) s[i] += talk_bias(size, rate, keys - 1 - min(key + i, keys - 1));
            s[i] = key + i < p.end ? s[i] : kScoredNone;
            top = fmaxf(top, s[i]);
        }
        const float next = fmaxf(m, top);
        l *= __builtin_amdgcn_exp2f(m - next);
        m = next;
#pragma unroll
        for (int i = 0; i < 4; ++i) l += key + i < p.end ? __builtin_amdgcn_exp2f(s[i] - m) : 0.f;
        if (l16 < n_heads && key < p.end) *reinterpret_cast<f4 *>(dst + key) = s;  // (keys_cap is a multiple of 64)
    };
    fetch(x[0], p.lo + 16 * wave + l16);
    for (int k0 = p.lo + 16 * wave; k0 < p.end; k0 += 2 * kTdKeys) {
        fetch(x[1], k0 + kTdKeys + l16);
        tile(x[0], k0);
        fetch(x[0], k0 + 2 * kTdKeys + l16);
        if (k0 + kTdKeys < p.end) tile(x[1], k0 + kTdKeys);
    }
    float top = fmaxf(m, __shfl_xor(m, 16, 64));
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    l *= __builtin_amdgcn_exp2f(m - top);
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g == 0) {
        ms[wave][l16] = top;
        ls[wave][l16] = l;
    }
    __syncthreads();
    if (tid < n_heads) {
        float all = ms[0][tid], sum = 0.f;
#pragma unroll
        for (int w = 1; w < 4; ++w) all = fmaxf(all, ms[w][tid]);
#pragma unroll
        for (int w = 0; w < 4; ++w) sum = fmaf(ls[w][tid], __builtin_amdgcn_exp2f(ms[w][tid] - all), sum);
        float *ml = a.part_ml + (((int64_t)b * a.heads + h0 + tid) * a.splits + piece) * 2;
        ml[0] = all;
        ml[1] = sum;
    }
}

// HP: heads padded to 32, 64 or 128 (the rows of P).
template <int VC, int HP> struct TdTile {
    static constexpr int vPitch = VC + 16, pPitch = kTdKeys + 8, vElems = kTdKeys * vPitch, pElems = HP * pPitch;
    static constexpr size_t bytes = (size_t)(vElems + 2 * pElems) * 2 + HP * 4;
};

template <int VC, int HP> __global__ __launch_bounds__(256) void talk_values_kernel(const TalkArgs a) {
    using L = TdTile<VC, HP>;
    constexpr int kVT = VC / 64, kVL = kTdKeys * VC / 8 / 256, kPL = HP * kTdKeys / 4 / 256, kSteps = HP / 32;
    extern __shared__ __align__(16) char td_lds[];
    __bf16 *vs = reinterpret_cast<__bf16 *>(td_lds), *p_hi = vs + L::vElems, *p_lo = p_hi + L::pElems;
    float *lse = reinterpret_cast<float *>(p_lo + L::pElems);
    const int groups = (a.n_rep + 15) / 16, kvh = blockIdx.x / groups, rep0 = blockIdx.x % groups * 16, piece = blockIdx.y, b = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const int keys = a.ctx_lens[b], h0 = kvh * a.n_rep + rep0, n_heads = min(16, a.n_rep - rep0);
    if (keys <= 0) return;  // padding
    const TdPiece p = td_piece(a, keys, piece);
    if (p.lo >= p.end) return;
    if (tid < HP) {
        float m = kScoredNone, l = 0.f;
        if (tid < a.heads) {
            const float *ml = a.part_ml + ((int64_t)b * a.heads + tid) * a.splits * 2;
            for (int s = 0; s < a.splits; ++s) {
                if (td_piece(a, keys, s).lo >= keys) break;
                const float next = fmaxf(m, ml[2 * s]);
                l = fmaf(l, __builtin_amdgcn_exp2f(m - next), ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - next));
                m = next;
            }
        }
        lse[tid] = m + __builtin_amdgcn_logf(l);
    }
    // T^T: out head l16, in heads 32 step + 8 g + j, as two terms
    bf8 t_hi[kSteps], t_lo[kSteps];
    bool exact = true;
#pragma unroll
    for (int st = 0; st < kSteps; ++st) {
        LaSplit sp;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            float x[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const int in = 32 * st + 8 * g + 2 * j + e;
                x[e] = l16 < n_heads && in < a.heads ? a.talk[(int64_t)(h0 + l16) * a.heads + in] : 0.f;
            }
            la_split2(x[0], x[1], sp.hi[j], sp.lo[j]);
            exact = exact && sp.lo[j] == 0;
        }
        t_hi[st] = sp.high();
        t_lo[st] = sp.low();
    }
    const bool t_rest = __ballot(!exact) != 0;  // (a matrix stored in 16 bits has no second term)
    const int32_t *table = a.bt + b * a.bt_stride;
    const uint16_t *vp = reinterpret_cast<const uint16_t *>(a.v) + (int64_t)kvh * a.v_dim;
    const int64_t v_tok = (int64_t)a.hkv * a.v_dim;
    const int vreal = (a.vdim + 7) / 8 * 8;
    const float *src = a.scores + (int64_t)b * a.heads * a.keys_cap;
    scored_u4 vr[kVL];
    f4 sr[kPL];
    auto id_of = [&](int k0) { return talk_block_id(a, table, min(k0 + lane, p.end - 1)); };
    auto fetch = [&](int id, int k0) {
        const int slots = talk_slot_of(a, id, k0 + lane, p.end);
#pragma unroll
        for (int n = 0; n < kVL; ++n) {
            const int c = tid + 256 * n, s = __shfl(slots, c / (VC / 8), 64), e = c % (VC / 8) * 8;
            vr[n] = scored_load16(vp + s * v_tok + e, s >= 0 && e < vreal);
        }
#pragma unroll
        for (int n = 0; n < kPL; ++n) {
            const int c = tid + 256 * n, h = min(c / 16, a.heads - 1);
            sr[n] = *reinterpret_cast<const f4 *>(src + h * a.keys_cap + min((int64_t)(k0 + c % 16 * 4), a.keys_cap - 4));
        }
    };
    f4 o[kVT];
#pragma unroll
    for (int c = 0; c < kVT; ++c) o[c] = f4{0.f, 0.f, 0.f, 0.f};
    fetch(id_of(p.lo), p.lo);
    int id = id_of(p.lo + kTdKeys);
    __syncthreads();  // (lse)
    for (int k0 = p.lo; k0 < p.end; k0 += kTdKeys) {
#pragma unroll
        for (int n = 0; n < kVL; ++n) {
            const int c = tid + 256 * n;
            *reinterpret_cast<scored_u4 *>(vs + c / (VC / 8) * L::vPitch + c % (VC / 8) * 8) = vr[n];
        }
#pragma unroll
        for (int n = 0; n < kPL; ++n) {
            const int c = tid + 256 * n, h = c / 16, key = c % 16 * 4;
            float w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) w[i] = h < a.heads && k0 + key + i < p.end ? __builtin_amdgcn_exp2f(sr[n][i] - lse[h]) : 0.f;
            uint2 hi, lo;
            la_split2(w[0], w[1], hi.x, lo.x);
            la_split2(w[2], w[3], hi.y, lo.y);
            *reinterpret_cast<uint2 *>(p_hi + h * L::pPitch + key) = hi;
            *reinterpret_cast<uint2 *>(p_lo + h * L::pPitch + key) = lo;
        }
        __syncthreads();
        if (k0 + kTdKeys < p.end) {
            fetch(id, k0 + kTdKeys);
            id = id_of(k0 + 2 * kTdKeys);
        }
        // mixed weights: keys 16 kt + 4 g + i of head l16
        uint2 w[4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
            f4 x = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int st = 0; st < kSteps; ++st) {
                const int at = (32 * st + 8 * g + (l16 >> 2)) * L::pPitch + 16 * kt + 4 * (l16 & 3);
                const bf8 hi = la_join(la_read_tr(p_hi + at), la_read_tr(p_hi + at + 4 * L::pPitch));
                const bf8 lo = la_join(la_read_tr(p_lo + at), la_read_tr(p_lo + at + 4 * L::pPitch));
                x = la_mfma(lo, t_hi[st], x);
                if (t_rest) x = la_mfma(hi, t_lo[st], x);
                x = la_mfma(hi, t_hi[st], x);
            }
            w[kt] = make_uint2(row_pack_bf16(x[0], x[1]), row_pack_bf16(x[2], x[3]));
        }
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const bf8 x = __builtin_bit_cast(bf8, la_u4{w[2 * kk].x, w[2 * kk].y, w[2 * kk + 1].x, w[2 * kk + 1].y});
#pragma unroll
            for (int c = 0; c < kVT; ++c) {
                const __bf16 *va = vs + (32 * kk + 4 * g + (l16 >> 2)) * L::vPitch + 16 * (wave * kVT + c) + 4 * (l16 & 3);
                o[c] = la_mfma(la_join(la_read_tr(va), la_read_tr(va + 16 * L::vPitch)), x, o[c]);
            }
        }
        __syncthreads();
    }
    if (l16 >= n_heads) return;
    const int64_t bh = (int64_t)b * a.heads + h0 + l16;
    if (a.splits > 1) {
        float *dst = a.part_o + (bh * a.splits + piece) * VC;
#pragma unroll
        for (int c = 0; c < kVT; ++c) *reinterpret_cast<f4 *>(dst + 16 * (wave * kVT + c) + 4 * g) = o[c];
        return;
    }
    pa_bf16 *dst = reinterpret_cast<pa_bf16 *>(a.out) + bh * a.vdim;
#pragma unroll
    for (int c = 0; c < kVT; ++c) {
        const int d = 16 * (wave * kVT + c) + 4 * g;
        if (d >= a.vdim) continue;
        if (a.vdim % 4 == 0) {
            *reinterpret_cast<uint2 *>(dst + d) = make_uint2(row_pack_bf16(o[c][0], o[c][1]), row_pack_bf16(o[c][2], o[c][3]));
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (d + i < a.vdim) pa_scalar<pa_bf16>::store(dst + d + i, o[c][i]);
        }
    }
}

// The parts of a sequence's pieces added up: four value columns per thread
__global__ __launch_bounds__(256) void talk_merge_kernel(const TalkArgs a, int vc) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, bh = i / (vc / 4);
    if (bh >= (int64_t)a.batch * a.heads) return;
    const int d = (int)(i % (vc / 4)) * 4, keys = a.ctx_lens[bh / a.heads];
    if (d >= a.vdim || keys <= 0) return;
    const float *src = a.part_o + bh * a.splits * vc + d;
    f4 sum = f4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.splits; ++s) {
        if (td_piece(a, keys, s).lo >= keys) break;
        const f4 x = *reinterpret_cast<const f4 *>(src + (int64_t)s * vc);
#pragma unroll
        for (int e = 0; e < 4; ++e) sum[e] += x[e];
    }
    pa_bf16 *out = reinterpret_cast<pa_bf16 *>(a.out) + bh * a.vdim + d;
    if (a.vdim % 4 == 0) {
        *reinterpret_cast<uint2 *>(out) = make_uint2(row_pack_bf16(sum[0], sum[1]), row_pack_bf16(sum[2], sum[3]));
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (d + e < a.vdim) pa_scalar<pa_bf16>::store(out + e, sum[e]);
    }
}

template <int VC, int HP> int launch_values(const TalkArgs &a, const dim3 &grid, hipStream_t s) {
    constexpr size_t lds = TdTile<VC, HP>::bytes;
    static_assert(lds <= 160 * 1024, "LDS of one compute unit");
    if (int rc = la_big_lds(talk_values_kernel<VC, HP>, lds, "pa_talking_attention")) return rc;
    talk_values_kernel<VC, HP><<<grid, dim3(256), lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_talking_attention (values)");
    return PA_OK;
}
template <int VC> int launch_values_heads(const TalkArgs &a, const dim3 &grid, hipStream_t s) {
    return a.heads <= 32 ? launch_values<VC, 32>(a, grid, s) : a.heads <= 64 ? launch_values<VC, 64>(a, grid, s) : launch_values<VC, 128>(a, grid, s);
}

int64_t td_keys_cap(int64_t max_keys) { return (max_keys + kTdKeys - 1) / kTdKeys * kTdKeys; }
int td_splits(int batch, int heads, int kv_heads, int64_t max_keys) {
    const int n = scored_splits((int64_t)batch * kv_heads * ((heads / kv_heads + 15) / 16), la_cus(), max_keys, false);
    return n > kTdMaxSplits ? kTdMaxSplits : n;
}
struct TdSpace {
    size_t scores, ml, parts;
};
TdSpace td_space(int batch, int heads, int vdim, int64_t max_keys, int splits) {
    const size_t bh = (size_t)batch * heads;
    return {bh * td_keys_cap(max_keys) * 4, (bh * splits * 2 * 4 + 255) / 256 * 256, splits > 1 ? bh * splits * td_value_cols(vdim) * 4 : 0};
}

}  // namespace

size_t pa_talking_decode_bytes(int batch, int heads, int kv_heads, int vdim, int64_t max_keys) {
    if (batch <= 0 || heads < kv_heads) return 0;
    const TdSpace n = td_space(batch, heads, vdim, max_keys, td_splits(batch, heads, kv_heads, max_keys));
    return n.scores + n.ml + n.parts;
}

bool pa_talking_decode_launch(const TalkArgs &in, int dtype, void *workspace, size_t workspace_bytes, hipStream_t s, int &rc) {
    TalkArgs a = in;
    const uintptr_t at = (uintptr_t)a.q1 | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)a.out;
    if (dtype != PA_BF16 || a.q_lens || (at & 15u) != 0 || a.n1 % 8 != 0 || a.k_dim % 8 != 0 || a.v_dim % 8 != 0 || a.q1_row % 8 != 0 ||
        a.q1_head % 8 != 0 || a.num_blocks * a.bs >= 0x7fffffff || a.bt_stride == 0 || !(a.scale > 0.f))
        return false;
    const int64_t max_keys = a.bt_stride * a.bs;
    a.splits = td_splits(a.batch, a.heads, a.hkv, max_keys);
    const TdSpace n = td_space(a.batch, a.heads, a.vdim, max_keys, a.splits);
    if (n.scores + n.ml + n.parts > workspace_bytes) return false;
    a.keys_cap = td_keys_cap(max_keys);
    a.scores = (float *)workspace;
    a.part_ml = (float *)((char *)workspace + n.scores);
    a.part_o = (float *)((char *)workspace + n.scores + n.ml);
    const dim3 grid((unsigned)(a.hkv * ((a.n_rep + 15) / 16)), (unsigned)a.splits, (unsigned)a.batch);
    if (a.n1 <= 64) talk_scores_kernel<64><<<grid, dim3(256), 0, s>>>(a);
    else if (a.n1 <= 128) talk_scores_kernel<128><<<grid, dim3(256), 0, s>>>(a);
    else talk_scores_kernel<256><<<grid, dim3(256), 0, s>>>(a);
    const int vc = td_value_cols(a.vdim);
    rc = [&]() -> int {
        PA_CHECK_LAUNCH("pa_talking_attention (scores)");
        if (int e = vc == 64 ? launch_values_heads<64>(a, grid, s) : vc == 128 ? launch_values_heads<128>(a, grid, s) : launch_values_heads<256>(a, grid, s)) return e;
        if (a.splits > 1) {
            const int64_t items = (int64_t)a.batch * a.heads * (vc / 4);
            talk_merge_kernel<<<dim3((unsigned)((items + 255) / 256)), dim3(256), 0, s>>>(a, vc);
            PA_CHECK_LAUNCH("pa_talking_attention (merge)");
        }
        return PA_OK;
    }();
    return true;
}
