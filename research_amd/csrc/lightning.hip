// Lightning attention: per head S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, with q, k, v = silu(projections) and
// S in 32-bit floats, kept per sequence in a pool of state slots.
//
// Two kernels.  The recurrent one (a decode step, and 32-bit prompts) reads the state once, walks its rows token by
// token in registers and writes the state once: HBM-bound on the state for one token.  The chunked one (16-bit
// prompts) multiplies 64 rows at a time on the matrix cores:
//     O = diag(decay^(t+1)) Q S + ((Q K^T) * decay^(t-s), s <= t) V
//     S = decay^64 S + K^T diag(decay^(63-s)) V
// The 32-bit factors of these products (S, the decayed scores, the decayed values) enter the bf16 matrix cores as a
// sum of two bf16 terms, which keeps 16 bits of their mantissa; q, k and v are bf16 to begin with.
//
// The state never leaves the registers of its wave between chunks: a wave owns a slice of the value columns, its
// accumulator tile [16 d][16 v] of S is, in register order, the B operand of Q S when the operand Q is read with the
// same order of d.
#include "linear_tiles.h"

namespace {

struct LaArgs {
    const void *u;  // [rows][ldu]: heads * dim of q, heads * dim of k, heads * vdim of v, anything
    int64_t ldu, n_rows;
    float *state;  // [state_rows][heads][pad16(dim)][pad16(vdim)]
    int64_t state_rows;
    const float *decay;  // [heads][kLaChunk + 1]: powers 0 .. 64 of a head's decay
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots;
    void *out;  // [rows][heads * vdim]
    float *ws;  // segment states
    int heads, dim, vdim, dp, vp;
    int segments, seg_rows;
};

// The portion of sequence b: rows [row0, row0 + n), the first at position pos0.  False: nothing to do.
struct Portion {
    int n, pos0;
    int64_t row0, slot;
};
__device__ __forceinline__ bool la_portion(const LaArgs &a, int b, Portion &p) {
    p.n = a.q_lens ? a.q_lens[b] : 1;
    p.row0 = a.q_starts ? a.q_starts[b] : b;
    p.pos0 = a.ctx_lens[b] - p.n;
    p.slot = a.state_slots[b];
    if (p.slot >= a.state_rows) p.slot = -1;
    return p.n > 0 && p.pos0 >= 0 && p.row0 >= 0 && p.row0 + p.n <= a.n_rows;
}

// ------------------------------------------------------------------ token by token
constexpr int kRecCols = 64;  // value columns per workgroup: 16 lanes x float4, 16 groups of lanes over the rows of S

// silu as the products of a layer see it: in the type of the activations
template <typename T> __device__ __forceinline__ float la_act(float x) {
    x = row_silu<T>(x);
    if constexpr (sizeof(T) == 2) return (float)(__bf16)x;
    return x;
}

// R: rows of S per thread (16 R >= dim)
template <typename T, int R> __global__ __launch_bounds__(256) void lightning_recurrent_kernel(const LaArgs a) {
    __shared__ float qs[16 * R], ks[16 * R], vs[kRecCols];
    __shared__ float4 red[16][kRecCols / 4];
    const int b = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * kRecCols;
    Portion p;
    if (!la_portion(a, b, p)) return;
    const int tid = threadIdx.x, col = tid % 16 * 4, grp = tid / 16;
    const bool live = v0 + col < a.vp;  // (vp is a multiple of 16)
    float *sp = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * (int64_t)a.dp * a.vp + v0 + col : nullptr;
    float4 s[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        s[r] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (sp && p.pos0 > 0 && live && d < a.dp) s[r] = *reinterpret_cast<const float4 *>(sp + (int64_t)d * a.vp);
    }
    const float lam = a.decay[h * (kLaChunk + 1) + 1];
    const T *u = reinterpret_cast<const T *>(a.u);
    for (int t = 0; t < p.n; ++t) {
        const T *row = u + (p.row0 + t) * a.ldu;
        for (int i = tid; i < 2 * 16 * R + kRecCols; i += 256) {
            if (i < 16 * R) {
                qs[i] = i < a.dim ? la_act<T>(pa_scalar<T>::load(row + h * a.dim + i)) : 0.f;
            } else if (i < 32 * R) {
                const int d = i - 16 * R;
                ks[d] = d < a.dim ? la_act<T>(pa_scalar<T>::load(row + (a.heads + h) * a.dim + d)) : 0.f;
            } else {
                const int v = i - 32 * R;
                vs[v] = v0 + v < a.vdim
                            ? la_act<T>(pa_scalar<T>::load(row + 2 * a.heads * a.dim + h * a.vdim + v0 + v)) : 0.f;
            }
        }
        __syncthreads();
        const float4 v = *reinterpret_cast<const float4 *>(vs + col);
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float k = ks[grp + 16 * r], q = qs[grp + 16 * r];
            s[r].x = fmaf(lam, s[r].x, k * v.x); s[r].y = fmaf(lam, s[r].y, k * v.y);
            s[r].z = fmaf(lam, s[r].z, k * v.z); s[r].w = fmaf(lam, s[r].w, k * v.w);
            o.x = fmaf(q, s[r].x, o.x); o.y = fmaf(q, s[r].y, o.y);
            o.z = fmaf(q, s[r].z, o.z); o.w = fmaf(q, s[r].w, o.w);
        }
        red[grp][tid % 16] = o;
        __syncthreads();
        if (tid < kRecCols && v0 + tid < a.vdim) {
            float sum = 0.f;
#pragma unroll
            for (int g = 0; g < 16; ++g) sum += reinterpret_cast<const float *>(red[g])[tid];
            pa_scalar<T>::store(reinterpret_cast<T *>(a.out) + (p.row0 + t) * ((int64_t)a.heads * a.vdim) + h * a.vdim + v0 + tid,
                                sum);
        }
        // (the next token's writes to qs, ks, vs follow every thread's reads of them, before the barrier above; its
        // writes to red come after its own barrier, which the threads that sum here reach afterwards)
    }
    if (!sp || !live) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        if (d < a.dp) *reinterpret_cast<float4 *>(sp + (int64_t)d * a.vp) = s[r];
    }
}

// ------------------------------------------------------------------ chunks on the matrix cores
// Elements of the tiles: Q and K row-major, the two terms of the decayed scores, the transposed K and V, the output.
template <int KD> constexpr int la_r_elems() { return 64 * (KD + 8); }
constexpr int kLaAElems = 2 * 64 * kLaPitchA;
template <int KD, int NW> constexpr int la_t_elems() { return (KD + 16 * NW) * 64; }
template <int NW> constexpr int la_o_elems() { return 64 * (16 * NW + 8); }
template <int KD, int NW, bool STATES> constexpr size_t la_lds_bytes() {
    const size_t elems = STATES ? 2 * la_t_elems<KD, NW>()  // (double-buffered: one barrier per chunk)
                                : 2 * la_r_elems<KD>() + kLaAElems + la_t_elems<KD, NW>() + la_o_elems<NW>();
    return elems * 2 + (64 + 64 + 64 + 80) * 4;
}

// KD: dim padded to 64, 128 or 256.  NW: waves; each owns 16 value columns.  All products are taken transposed (value
// columns, or keys, as the rows of the result), so that a lane holds four consecutive elements of one row t.
// STATES: only the segment's own contribution to the state, to the workspace (first pass over a portion in segments).
template <int KD, int NW, bool STATES>
__global__ __launch_bounds__(64 * NW, 2) void lightning_chunk_kernel(const LaArgs a) {
    constexpr int kCols = 16 * NW, kLdR = KD + 8, kLdO = kCols + 8, kThr = 64 * NW;
    constexpr int kDB = KD / 4, kKBlocks = 16 * kDB, kKPass = (kKBlocks + kThr - 1) / kThr;  // 4x4 blocks of K
    constexpr int kST = NW == 8 ? 2 : 4;  // score tiles per wave
    extern __shared__ __align__(16) char lds[];
    float *rev = reinterpret_cast<float *>(lds);  // decay from row s to the last row of a whole chunk ...
    float *rev_tail = rev + 64;                   // ... and of a portion's last chunk
    float *pw = rev + 192;                        // powers 0 .. 64, behind 64 zeros for the keys after a row
    __bf16 *tiles = reinterpret_cast<__bf16 *>(rev + 272);
    __bf16 *kt_s = tiles, *vt_s = kt_s + KD * 64;
    __bf16 *q_s = tiles + la_t_elems<KD, NW>(), *k_s = q_s + la_r_elems<KD>(), *a_hi = k_s + la_r_elems<KD>();
    __bf16 *a_lo = a_hi + 64 * kLaPitchA, *o_s = a_hi + kLaAElems;

    const int h = blockIdx.x, seg = blockIdx.y % a.segments, vsl = blockIdx.y / a.segments, b = blockIdx.z;
    Portion p;
    if (!la_portion(a, b, p)) return;
    const int r_beg = seg * a.seg_rows, r_end = r_beg + a.seg_rows < p.n ? r_beg + a.seg_rows : p.n;
    if (r_beg >= p.n) return;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = vsl * kCols, vw = wave * 16;  // first column of the workgroup, of the wave inside it
    const float *powers = a.decay + h * (kLaChunk + 1);
    if (tid <= kLaChunk) pw[tid] = powers[tid];
    if (tid < 64) {
        rev[tid] = powers[63 - tid];
        pw[tid - 64] = 0.f;
    }
    const int l16 = tid & 15, g = (tid & 63) >> 4;
    float pt[4];  // decay from the chunk's start to row 16 tt + l16
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) pt[tt] = powers[16 * tt + l16 + 1];

    // The state slice of this wave: tile dt holds d = 16 dt + 4 g + i, v = v0 + vw + l16
    f4 s[KD / 16];
    const int64_t state_elems = (int64_t)a.dp * a.vp;
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * state_elems : nullptr;
    float *seg_state = a.segments > 1 ? a.ws + (((int64_t)b * a.heads + h) * a.segments + seg) * state_elems : nullptr;
    const float *from = STATES ? nullptr : (a.segments > 1 ? seg_state : (p.pos0 > 0 ? pool : nullptr));
    // (a state as a buffer: rows past dp lie past its end, columns past vp get an offset outside)
    const int state_bytes = (int)state_elems * 4;
    const int v = v0 + vw + l16;
    const uint32_t soff = v < a.vp ? (uint32_t)(4 * g * a.vp + v) * 4u : kLaOutside;
    {
        const __amdgpu_buffer_rsrc_t src = __builtin_amdgcn_make_buffer_rsrc(
            (void *)(from ? from : a.state), 0, from ? state_bytes : 0, 0x00020000);  // (no state: every load is past the end)
#pragma unroll
        for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                s[dt][i] = __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(src, soff + (16 * dt + i) * a.vp * 4, 0, 0));
    }

    const uint16_t *u = reinterpret_cast<const uint16_t *>(a.u) + p.row0 * a.ldu;
    const uint16_t *uq = u + h * a.dim, *uk = u + (a.heads + h) * a.dim;
    const uint16_t *uv = u + 2 * a.heads * a.dim + h * a.vdim + v0;
    const int vcols = a.vdim - v0 < kCols ? a.vdim - v0 : kCols;
    const uint32_t row_bytes = (uint32_t)a.ldu * 2u;
    LaBlock kb[kKPass], qb[STATES ? 1 : kKPass], vb;
    uint32_t koff[kKPass];
#pragma unroll
    for (int i = 0; i < kKPass; ++i) {
        const int blk = tid + kThr * i;
        koff[i] = blk < kKBlocks ? la_block_off(a.ldu, blk / kDB * 4, blk % kDB * 4, a.dim) : kLaOutside;
    }
    const uint32_t voff = la_block_off(a.ldu, tid / (kCols / 4) * 4, tid % (kCols / 4) * 4, vcols);
    auto fetch = [&](int r0) {
        const int rows = r_end - r0 < kLaChunk ? r_end - r0 : kLaChunk;
        const int64_t at = (int64_t)r0 * a.ldu;
        const __amdgpu_buffer_rsrc_t tk = la_tile(uk + at, a.ldu, rows, a.dim), tv = la_tile(uv + at, a.ldu, rows, vcols);
        if (!STATES) {
            const __amdgpu_buffer_rsrc_t tq = la_tile(uq + at, a.ldu, rows, a.dim);
#pragma unroll
            for (int i = 0; i < kKPass; ++i) qb[i] = la_load_block(tq, koff[i], row_bytes);
        }
#pragma unroll
        for (int i = 0; i < kKPass; ++i) kb[i] = la_load_block(tk, koff[i], row_bytes);
        vb = la_load_block(tv, voff, row_bytes);
    };
    fetch(r_beg);
    for (int r0 = r_beg; r0 < r_end; r0 += kLaChunk) {
        const int nv = r_end - r0 < kLaChunk ? r_end - r0 : kLaChunk;
#pragma unroll
        for (int i = 0; i < kKPass; ++i) {
            const int blk = tid + kThr * i, c = blk % kDB * 4, sr = blk / kDB * 4;
            if (kKBlocks % kThr != 0 && blk >= kKBlocks) continue;
            la_put_block<true>(kb[i], sr, c, STATES ? nullptr : k_s, kLdR, kt_s);
            if (!STATES) la_put_block<true>(qb[i], sr, c, q_s, kLdR, nullptr);
        }
        la_put_block<true>(vb, tid / (kCols / 4) * 4, tid % (kCols / 4) * 4, nullptr, 0, vt_s);
        if (nv < kLaChunk && tid < 64) rev_tail[tid] = tid < nv ? powers[nv - 1 - tid] : 0.f;
        if (r0 + kLaChunk < r_end) fetch(r0 + kLaChunk);
        __syncthreads();

        f4 o[4];  // O^T: v = 4 g + i of the wave's columns, t = 16 tt + l16
        if constexpr (!STATES) {
            // score tiles (st, rt): keys 16 st + 4 g + i, rows 16 rt + l16
            const int rt = NW == 8 ? wave >> 1 : wave;
            f4 sc[kST];
#pragma unroll
            for (int m = 0; m < kST; ++m) sc[m] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KD / 32; ++kk) {
                const bf8 bq = la_read8(q_s + (16 * rt + l16) * kLdR + 32 * kk + 8 * g);
#pragma unroll
                for (int m = 0; m < kST; ++m) {
                    const int st = NW == 8 ? 2 * m + (wave & 1) : m;
                    if (st <= rt) sc[m] = la_mfma(la_read8(k_s + (16 * st + l16) * kLdR + 32 * kk + 8 * g), bq, sc[m]);
                }
            }
            // the rows' part from before the chunk: Q S, then the decay of the way from the chunk's start
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) o[tt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int dd = 0; dd < KD / 32; ++dd) {
                LaSplit sp;
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    la_split2(s[2 * dd + j / 2][2 * j % 4], s[2 * dd + j / 2][2 * j % 4 + 1], sp.hi[j], sp.lo[j]);
                const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
                for (int tt = 0; tt < 4; ++tt) {
                    const __bf16 *qr = q_s + (16 * tt + l16) * kLdR + 32 * dd + 4 * g;
                    const bf8 bq = la_read44(qr, qr + 16);
                    o[tt] = la_mfma(hi, bq, o[tt]);
                    o[tt] = la_mfma(lo, bq, o[tt]);
                }
            }
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)
#pragma unroll
                for (int i = 0; i < 4; ++i) o[tt][i] *= pt[tt];
#pragma unroll
            for (int m = 0; m < kST; ++m) {
                const int st = NW == 8 ? 2 * m + (wave & 1) : m;
                if (st > rt + 1) continue;  // (tile rt + 1 is read as zeros when the last k-step covers it)
                const int t = 16 * rt + l16, c = 16 * st + 4 * g;
                const float *f = pw + t - c;
                uint2 hi, lo;
                la_split2(sc[m][0] * f[0], sc[m][1] * f[-1], hi.x, lo.x);
                la_split2(sc[m][2] * f[-2], sc[m][3] * f[-3], hi.y, lo.y);
                *reinterpret_cast<uint2 *>(a_hi + t * kLaPitchA + c) = hi;
                *reinterpret_cast<uint2 *>(a_lo + t * kLaPitchA + c) = lo;
            }
            __syncthreads();
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                const bf8 av = la_read8(vt_s + la_tr(vw + l16, 32 * kk + 8 * g));
#pragma unroll
                for (int tt = 2 * kk; tt < 4; ++tt) {
                    o[tt] = la_mfma(av, la_read8(a_hi + (16 * tt + l16) * kLaPitchA + 32 * kk + 8 * g), o[tt]);
                    o[tt] = la_mfma(av, la_read8(a_lo + (16 * tt + l16) * kLaPitchA + 32 * kk + 8 * g), o[tt]);
                }
            }
#pragma unroll
            for (int tt = 0; tt < 4; ++tt)  // to LDS, so that rows are stored 16 bytes per lane
                *reinterpret_cast<uint2 *>(o_s + (16 * tt + l16) * kLdO + vw + 4 * g) =
                    make_uint2(row_pack_bf16(o[tt][0], o[tt][1]), row_pack_bf16(o[tt][2], o[tt][3]));
        }
        // S <- decay^nv S + K^T (decay^(nv-1-s) V)
        const float whole = pw[nv];
        const float *wt = nv < kLaChunk ? rev_tail : rev;
#pragma unroll
        for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i) s[dt][i] *= whole;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            LaSplit sp;
            const la_u4 bv = *reinterpret_cast<const la_u4 *>(vt_s + la_tr(vw + l16, 32 * kk + 8 * g));
            const f4 w0 = *reinterpret_cast<const f4 *>(wt + 32 * kk + 8 * g);
            const f4 w1 = *reinterpret_cast<const f4 *>(wt + 32 * kk + 8 * g + 4);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const uint32_t pair = bv[j];
                la_split2(__builtin_bit_cast(float, pair << 16) * (j < 2 ? w0 : w1)[2 * j % 4],
                          __builtin_bit_cast(float, pair & 0xffff0000u) * (j < 2 ? w0 : w1)[2 * j % 4 + 1], sp.hi[j], sp.lo[j]);
            }
            const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
            for (int dt = 0; dt < KD / 16; ++dt) {
                const bf8 ak = la_read8(kt_s + la_tr(16 * dt + l16, 32 * kk + 8 * g));
                s[dt] = la_mfma(ak, hi, s[dt]);
                s[dt] = la_mfma(ak, lo, s[dt]);
            }
        }
        if constexpr (!STATES) {
            __syncthreads();
            const int ldo = a.heads * a.vdim;
            const uint16_t *first = reinterpret_cast<const uint16_t *>(a.out) + (p.row0 + r0) * (int64_t)ldo + h * a.vdim + v0;
            const __amdgpu_buffer_rsrc_t dst = la_tile(first, ldo, nv, vcols);
#pragma unroll
            for (int i = 0; i < 2; ++i) {  // (64 rows of kCols columns are two 16-byte vectors per thread)
                const int vec = tid + kThr * i, t = vec / (kCols / 8), c = vec % (kCols / 8) * 8;
                const la_u4 x = *reinterpret_cast<const la_u4 *>(o_s + t * kLdO + c);
                __builtin_amdgcn_raw_buffer_store_b128(x, dst, c < vcols ? (uint32_t)(t * ldo + c) * 2u : kLaOutside, 0, 0);
            }
            // (the next chunk's tiles may be written now: their readers are past the barrier above, and its scores and
            // output come behind barriers of its own)
        } else {  // the other half of the tiles
            kt_s = kt_s == tiles ? tiles + la_t_elems<KD, NW>() : tiles;
            vt_s = kt_s + KD * 64;
        }
    }
    float *to = STATES ? seg_state : (a.segments > 1 ? nullptr : pool);
    if (!to) return;
    const __amdgpu_buffer_rsrc_t dst = __builtin_amdgcn_make_buffer_rsrc((void *)to, 0, state_bytes, 0x00020000);
    uint32_t base = soff;
    asm volatile("" : "+v"(base));  // (offsets made again here instead of kept in registers over the loop)
#pragma unroll
    for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float f = s[dt][i];
            __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(uint32_t, f), dst, base + (16 * dt + i) * a.vp * 4, 0, 0);
        }
}

// Segment contributions -> start states, in place; the state after the last segment goes back to the pool.
__global__ __launch_bounds__(256) void lightning_scan_kernel(const LaArgs a) {
    const int h = blockIdx.y, b = blockIdx.z;
    Portion p;
    if (!la_portion(a, b, p)) return;
    const int64_t n4 = (int64_t)a.dp * a.vp / 4, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n4) return;
    float4 *pool = p.slot >= 0 ? reinterpret_cast<float4 *>(a.state) + (p.slot * a.heads + h) * n4 + i : nullptr;
    float4 *seg = reinterpret_cast<float4 *>(a.ws) + ((int64_t)b * a.heads + h) * a.segments * n4 + i;
    float4 cur = pool && p.pos0 > 0 ? *pool : make_float4(0.f, 0.f, 0.f, 0.f);
    const float *pw = a.decay + h * (kLaChunk + 1);
    float whole = 1.f;  // decay^seg_rows, seg_rows a multiple of the chunk
    for (int c = 0; c < a.seg_rows / kLaChunk; ++c) whole *= pw[kLaChunk];
    for (int j = 0; j * a.seg_rows < p.n; ++j) {
        float f = whole;
        const int left = p.n - j * a.seg_rows;
        if (left < a.seg_rows) {
            f = pw[left % kLaChunk];
            for (int c = 0; c < left / kLaChunk; ++c) f *= pw[kLaChunk];
        }
        const float4 add = seg[j * n4];
        seg[j * n4] = cur;
        cur = make_float4(fmaf(f, cur.x, add.x), fmaf(f, cur.y, add.y), fmaf(f, cur.z, add.z), fmaf(f, cur.w, add.w));
    }
    if (pool) *pool = cur;
}

template <int KD, int NW> int launch_chunks(const LaArgs &a, int batch, hipStream_t s) {
    constexpr size_t lds = la_lds_bytes<KD, NW, false>(), lds_states = la_lds_bytes<KD, NW, true>();
    static_assert(lds <= 160 * 1024 && lds_states <= 160 * 1024, "LDS of one compute unit");
    const int slices = (a.vdim + 16 * NW - 1) / (16 * NW);
    const dim3 grid((unsigned)a.heads, (unsigned)(slices * a.segments), (unsigned)batch), block(64 * NW);
    if (a.segments > 1) {
        if (int rc = la_big_lds(lightning_chunk_kernel<KD, NW, true>, lds_states, "pa_lightning_chunked")) return rc;
        lightning_chunk_kernel<KD, NW, true><<<grid, block, lds_states, s>>>(a);
        const unsigned gx = (unsigned)(((int64_t)a.dp * a.vp / 4 + 255) / 256);
        lightning_scan_kernel<<<dim3(gx, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s>>>(a);
    }
    if (int rc = la_big_lds(lightning_chunk_kernel<KD, NW, false>, lds, "pa_lightning_chunked")) return rc;
    lightning_chunk_kernel<KD, NW, false><<<grid, block, lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_lightning_chunked");
    return PA_OK;
}

template <typename T> void launch_recurrent(const LaArgs &a, int batch, hipStream_t s) {
    const dim3 grid((unsigned)batch, (unsigned)a.heads, (unsigned)((a.vdim + kRecCols - 1) / kRecCols)), block(256);
    if (a.dim <= 64) lightning_recurrent_kernel<T, 4><<<grid, block, 0, s>>>(a);
    else if (a.dim <= 128) lightning_recurrent_kernel<T, 8><<<grid, block, 0, s>>>(a);
    else lightning_recurrent_kernel<T, 16><<<grid, block, 0, s>>>(a);
}

int la_fill(const char *what, LaArgs &a, const void *u, int64_t u_stride, int64_t n_rows, float *state, int64_t state_rows,
            const float *decay_powers, const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
            const int32_t *state_slots, int batch, void *out, int num_heads, int dim, int vdim, int dtype) {
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && state_rows >= 0, "%s: a count is negative", what);
    PA_REQUIRE(num_heads > 0 && dim > 0 && vdim > 0, "%s: heads / dim / vdim must be positive", what);
    PA_REQUIRE(num_heads <= 65535 && batch <= 65535, "%s: heads=%d / batch=%d above 65535", what, num_heads, batch);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "%s: dtype=%d is not F32 or BF16", what, dtype);
    if (dim > 256) return pa_fail(PA_ERR_UNSUPPORTED, "%s: dim=%d above 256", what, dim);
    PA_REQUIRE(u_stride >= (int64_t)num_heads * (2 * dim + vdim), "%s: u_stride=%lld is shorter than q, k and v", what,
               (long long)u_stride);
    PA_REQUIRE((int64_t)num_heads * (2 * dim + vdim) <= 0x7fffffff, "%s: rows are too long", what);
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "%s: q_lens and q_starts come together", what);
    if (n_rows == 0 || batch == 0) return PA_OK;
    PA_REQUIRE(u && state && decay_powers && ctx_lens && state_slots && out, "%s: NULL argument", what);
    PA_REQUIRE(pa_aligned16(state), "%s: the state must be 16-byte aligned", what);
    a = LaArgs{};
    a.u = u; a.ldu = u_stride; a.n_rows = n_rows; a.state = state; a.state_rows = state_rows; a.decay = decay_powers;
    a.ctx_lens = ctx_lens; a.q_lens = q_lens; a.q_starts = q_starts; a.state_slots = state_slots; a.out = out;
    a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.dp = la_pad16(dim); a.vp = la_pad16(vdim);
    a.segments = 1;
    return PA_OK;
}

int la_plan(int64_t batch, int heads, int dim, int vdim, int max_q_len) {
    (void)dim;
    const int cols = la_value_cols(vdim);
    return la_segments(batch * heads * ((vdim + cols - 1) / cols), la_cus(), max_q_len);
}

}  // namespace

extern "C" size_t pa_lightning_state_floats(int dim, int vdim) {
    return dim > 0 && vdim > 0 ? la_state_floats(dim, vdim) : 0;
}

extern "C" int pa_lightning_recurrent(const void *u, int64_t u_stride, int64_t n_rows, float *state, int64_t state_rows,
                                      const float *decay_powers, const int32_t *ctx_lens, const int32_t *q_lens,
                                      const int32_t *q_starts, const int32_t *state_slots, int batch, void *out,
                                      int num_heads, int dim, int vdim, int dtype, void *stream) {
    pa_clear_error();
    LaArgs a;
    if (int rc = la_fill("pa_lightning_recurrent", a, u, u_stride, n_rows, state, state_rows, decay_powers, ctx_lens, q_lens,
                         q_starts, state_slots, batch, out, num_heads, dim, vdim, dtype))
        return rc;
    if (n_rows == 0 || batch == 0) return PA_OK;
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    if (dtype == PA_F32) launch_recurrent<float>(a, batch, (hipStream_t)stream);
    else launch_recurrent<pa_bf16>(a, batch, (hipStream_t)stream);
    PA_CHECK_LAUNCH("pa_lightning_recurrent");
    return PA_OK;
}

extern "C" size_t pa_lightning_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len) {
    pa_clear_error();
    if (batch < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || max_q_len < 0) {
        pa_fail(PA_ERR_INVALID_ARG, "pa_lightning_workspace_bytes: sizes out of range");
        return 0;
    }
    return la_workspace_bytes(batch, num_heads, dim, vdim, la_plan(batch, num_heads, dim, vdim, max_q_len));
}

extern "C" int pa_lightning_chunked(const void *u, int64_t u_stride, int64_t n_rows, float *state, int64_t state_rows,
                                    const float *decay_powers, const int32_t *ctx_lens, const int32_t *q_lens,
                                    const int32_t *q_starts, const int32_t *state_slots, int batch, int max_q_len,
                                    void *out, int num_heads, int dim, int vdim, int dtype, void *workspace,
                                    size_t workspace_bytes, void *stream) {
    pa_clear_error();
    LaArgs a;
    PA_REQUIRE(max_q_len >= 0, "max_q_len=%d is negative", max_q_len);
    if (dtype != PA_BF16)
        return pa_fail(PA_ERR_UNSUPPORTED, "pa_lightning_chunked: dtype=%d is not BF16 (32-bit rows take pa_lightning_recurrent)",
                       dtype);
    if (int rc = la_fill("pa_lightning_chunked", a, u, u_stride, n_rows, state, state_rows, decay_powers, ctx_lens, q_lens,
                         q_starts, state_slots, batch, out, num_heads, dim, vdim, dtype))
        return rc;
    if (n_rows == 0 || batch == 0 || max_q_len == 0) return PA_OK;
    PA_REQUIRE(q_lens, "NULL q_lens / q_starts");
    a.segments = la_plan(batch, num_heads, dim, vdim, max_q_len);
    while (a.segments > 1 && (!workspace || la_workspace_bytes(batch, num_heads, dim, vdim, a.segments) > workspace_bytes))
        --a.segments;
    a.seg_rows = la_segment_rows(max_q_len, a.segments);
    a.ws = (float *)workspace;
    PA_REQUIRE(a.segments == 1 || pa_aligned16(workspace), "the workspace must be 16-byte aligned");
    hipStream_t s = (hipStream_t)stream;
    // rows that are not whole 16-byte vectors, or too far apart for a tile's 32-bit offsets: token by token
    if (dim % 8 != 0 || vdim % 8 != 0 || u_stride % 8 != 0 || !pa_aligned16(u) || !pa_aligned16(out) ||
        u_stride > (1 << 22) || (int64_t)num_heads * vdim > (1 << 22)) {
        launch_recurrent<pa_bf16>(a, batch, s);
        PA_CHECK_LAUNCH("pa_lightning_chunked");
        return PA_OK;
    }
    const bool wide = la_value_cols(vdim) == 128;
    if (dim <= 64) return wide ? launch_chunks<64, 8>(a, batch, s) : launch_chunks<64, 4>(a, batch, s);
    if (dim <= 128) return wide ? launch_chunks<128, 8>(a, batch, s) : launch_chunks<128, 4>(a, batch, s);
    return wide ? launch_chunks<256, 8>(a, batch, s) : launch_chunks<256, 4>(a, batch, s);
}
