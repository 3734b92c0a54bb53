// Linear attention whose forget gate has a factor per channel and also decides what is written (HGRN2): per head
//     f_t = lower + (1 - lower) sigmoid(z_t + bias),   S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,   o_t = S_t^T q_t
// with S in 32-bit floats, kept per sequence in a pool of state slots.
//
// The recurrent kernel (a decode step, and 32-bit prompts) reads the state once, walks its rows token by token in registers
// and writes the state once.  The chunked one (16-bit prompts) works in blocks of 16 rows.  With P_t the product of the
// block's factors up to t, R_t the product of those behind t and B = P of the last row, all per channel,
//     O = (P Q) S + tril((P Q) (K / P)^T) V,   S <- diag(B) S + (R K)^T V,   K = 1 - f
// on the matrix cores, every 32-bit factor as a sum of two bf16 terms.  P and R are plain products, so no logarithm is taken
// and nothing overflows, except 1 / P where a channel forgets nearly everything inside a block: such a block's scores are
// taken token by token.
#include "linear_tiles.h"

namespace {

struct ClArgs {
    const void *q, *z, *v;  // row strides ldq, ldz, ldv; head h: q, z at h * dim, v at h * vdim
    int64_t ldq, ldz, ldv;
    const float *bias, *lower;  // [heads * dim] (bias: or NULL)
    int silu;                   // q's activation
    int64_t n_rows;
    float *state;  // [state_rows][heads][dp][vp]
    int64_t state_rows;
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots;
    void *out;  // [rows][heads * vdim]
    float *ws;  // segment states: S [dp][vp], the segment's factors [dp], padding
    int heads, dim, vdim, dp, vp;
    int segments, seg_rows;
};

struct ClPortion {
    int n, pos0;
    int64_t row0, slot;
};
__device__ __forceinline__ bool cl_portion(const ClArgs &a, int b, ClPortion &p) {
    p.n = a.q_lens ? a.q_lens[b] : 1;
    p.row0 = a.q_starts ? a.q_starts[b] : b;
    p.pos0 = a.ctx_lens[b] - p.n;
    p.slot = a.state_slots[b];
    if (p.slot >= a.state_rows) p.slot = -1;
    return p.n > 0 && p.pos0 >= 0 && p.row0 >= 0 && p.row0 + p.n <= a.n_rows;
}

// f and 1 - f, neither by subtraction from one
template <typename T> __device__ __forceinline__ void cl_gate(float z, float lower, float &f, float &k) {
    float e, big;
    if constexpr (sizeof(T) == 4) {
        e = expf(-fabsf(z));
        big = 1.f / (1.f + e);
    } else {
        e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
        big = __builtin_amdgcn_rcpf(1.f + e);
    }
    const float small = e * big, open = 1.f - lower;
    f = fmaf(open, z >= 0.f ? big : small, lower);
    k = open * (z >= 0.f ? small : big);
}

// ------------------------------------------------------------------ token by token
constexpr int kClCols = 64;  // value columns per workgroup: 16 lanes x float4, 16 groups of lanes over the rows of S

// R: rows of S per thread (16 R >= dim).
template <typename T, int R> __global__ __launch_bounds__(256, 4) void channel_recurrent_kernel(const ClArgs a) {
    __shared__ float qs[2][16 * R], fs[2][16 * R], ks[2][16 * R], vs[2][kClCols];
    __shared__ float4 red[16][kClCols / 4];
    const int h = blockIdx.y, b = blockIdx.z, v0 = blockIdx.x * kClCols;
    ClPortion p;
    if (!cl_portion(a, b, p)) return;
    const int tid = threadIdx.x, col = tid % 16 * 4, grp = tid / 16;
    const bool live = v0 + col < a.vp;  // (vp is a multiple of 16)
    float *head = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * ((int64_t)a.dp * a.vp) : nullptr;
    float *sp = head ? head + v0 + col : nullptr;
    const bool resume = head && p.pos0 > 0;
    float4 s[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        s[r] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (resume && live && d < a.dp) s[r] = *reinterpret_cast<const float4 *>(sp + (int64_t)d * a.vp);
    }
    const T *q = reinterpret_cast<const T *>(a.q) + h * a.dim, *z = reinterpret_cast<const T *>(a.z) + h * a.dim;
    const T *v = reinterpret_cast<const T *>(a.v) + h * a.vdim + v0;
    for (int t = 0; t < p.n; ++t) {
        const int64_t row = p.row0 + t;
        const int at = t & 1;
        for (int i = tid; i < 2 * 16 * R + kClCols; i += 256) {
            if (i < 16 * R) {
                float x = i < a.dim ? pa_scalar<T>::load(q + row * a.ldq + i) : 0.f;
                qs[at][i] = a.silu ? row_silu<T>(x) : x;
            } else if (i < 32 * R) {
                const int d = i - 16 * R;
                float f = 1.f, k = 0.f;
                if (d < a.dim) {
                    const int c = h * a.dim + d;
                    cl_gate<T>(pa_scalar<T>::load(z + row * a.ldz + d) + (a.bias ? a.bias[c] : 0.f), a.lower[c], f, k);
                }
                fs[at][d] = f;
                ks[at][d] = k;
            } else {
                const int c = i - 32 * R;
                vs[at][c] = v0 + c < a.vdim ? pa_scalar<T>::load(v + row * a.ldv + c) : 0.f;
            }
        }
        __syncthreads();
        const float4 x = *reinterpret_cast<const float4 *>(vs[at] + col);
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float f = fs[at][grp + 16 * r], k = ks[at][grp + 16 * r], qd = qs[at][grp + 16 * r];
            s[r].x = fmaf(f, s[r].x, k * x.x); s[r].y = fmaf(f, s[r].y, k * x.y);
            s[r].z = fmaf(f, s[r].z, k * x.z); s[r].w = fmaf(f, s[r].w, k * x.w);
            o.x = fmaf(qd, s[r].x, o.x); o.y = fmaf(qd, s[r].y, o.y);
            o.z = fmaf(qd, s[r].z, o.z); o.w = fmaf(qd, s[r].w, o.w);
        }
        red[grp][tid % 16] = o;
        __syncthreads();
        if (tid < kClCols && v0 + tid < a.vdim) {
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) sum += reinterpret_cast<const float *>(red[i])[tid];
            pa_scalar<T>::store(reinterpret_cast<T *>(a.out) + row * ((int64_t)a.heads * a.vdim) + h * a.vdim + v0 + tid, sum);
        }
        // (the next token writes the other half of qs .. vs; its writes to red come after its own barrier, which the threads
        // that sum here reach afterwards)
    }
    if (!head) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        if (live && d < a.dp) *reinterpret_cast<float4 *>(sp + (int64_t)d * a.vp) = s[r];
    }
}

// ------------------------------------------------------------------ blocks on the matrix cores
constexpr int kClBlock = 16;
constexpr float kClSmall = 0x1p-100f;  // a block whose P falls below has its scores taken token by token

// KD: dim padded to 64, 128 or 256.  NW: waves; each owns 16 value columns.
template <int KD, int NW, bool STATES> struct ClTile {
    static constexpr int rows = KD == 256 ? 32 : 64, blocks = rows / kClBlock, cols = 16 * NW, threads = 64 * NW;
    static constexpr int pitch = KD + 8, vPitch = cols + 8;
    static constexpr int elems = rows * pitch;                       // one bf16 term of a tile
    static constexpr int units = KD / 2 * rows / 8;                  // (channel pair, 8 rows)
    static constexpr int passes = (units + threads - 1) / threads;
    static constexpr int vLoads = rows * cols / 4 / threads;         // four columns each
    static constexpr size_t bytes = (size_t)elems * (STATES ? 2 : 6) * 2 + (size_t)rows * vPitch * 2 + (size_t)blocks * KD * 4 +
                                    (STATES ? 0 : (size_t)blocks * 64 * 16) + 64;
};

// Scores of one block token by token, a wave: a lane follows its channels' k_s f_(s+1) .. f_t for all s in `follow` (16 rows
// of KD floats, the block's part of the K / P tiles: rows 0 .. 7 and 8 .. 15 apart).  Returns scores s = 4 g + i of row l16.
// (Out of line, and its arguments one by one: it is rarely called, and must not put the kernel's into memory.)
template <int KD> __device__ __noinline__ f4 cl_slow_scores(const uint16_t *uq, int64_t ldq, const uint16_t *uz, int64_t ldz, const float *bias,
                                                            const float *lower, int dim, int silu, int n_rows, float *lo8, float *hi8) {
    const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
    f4 out = f4{0.f, 0.f, 0.f, 0.f};
    auto at = [&](int s) { return (s < 8 ? lo8 : hi8) + (s & 7) * KD; };
    for (int t = 0; t < n_rows; ++t) {
        float part[kClBlock];
#pragma unroll
        for (int s = 0; s < kClBlock; ++s) part[s] = 0.f;
        for (int d = lane; d < dim; d += 64) {
            float q = pa_scalar<pa_bf16>::load(reinterpret_cast<const pa_bf16 *>(uq) + t * ldq + d), f, k;
            if (silu) q = row_silu<pa_bf16>(q);
            cl_gate<pa_bf16>(pa_scalar<pa_bf16>::load(reinterpret_cast<const pa_bf16 *>(uz) + t * ldz + d) + (bias ? bias[d] : 0.f), lower[d], f, k);
#pragma unroll
            for (int s = 0; s < kClBlock; ++s) {
                if (s > t) continue;
                float *w = at(s) + d;
                const float x = s == t ? k : *w * f;
                *w = x;
                part[s] = fmaf(q, x, part[s]);
            }
        }
#pragma unroll
        for (int s = 0; s < kClBlock; ++s) {
            const float sum = pa_group_sum<64>(part[s]);
            if (l16 == t && g == s / 4) out[s % 4] = s <= t ? sum : 0.f;
        }
    }
    return out;
}

// STATES: only the segment's own contribution to the state and its factors, to the workspace (first pass over a portion in
// segments).
template <int KD, int NW, bool STATES>
__global__ __launch_bounds__(64 * NW, 1) void channel_chunk_kernel(const ClArgs a) {
    using L = ClTile<KD, NW, STATES>;
    constexpr int kRows = L::rows, kPitch = L::pitch, kThr = L::threads, kPairs = KD / 2;
    extern __shared__ __align__(16) char lds[];
    __bf16 *k_hi = reinterpret_cast<__bf16 *>(lds), *k_lo = k_hi + L::elems;         // R K
    __bf16 *q_hi = k_lo + L::elems, *q_lo = q_hi + L::elems;                         // P Q
    __bf16 *i_hi = q_lo + L::elems, *i_lo = i_hi + L::elems;                         // K / P
    __bf16 *v_s = STATES ? q_hi : i_lo + L::elems;
    float *whole = reinterpret_cast<float *>(v_s + kRows * L::vPitch);               // B per block
    uint4 *scores = reinterpret_cast<uint4 *>(whole + L::blocks * KD);               // per block and lane: four scores, two terms
    int *unsafe = reinterpret_cast<int *>(STATES ? scores : scores + L::blocks * 64);

    const int h = blockIdx.x, seg = blockIdx.y % a.segments, vsl = blockIdx.y / a.segments, b = blockIdx.z;
    ClPortion p;
    if (!cl_portion(a, b, p)) return;
    const int r_beg = seg * a.seg_rows, r_end = r_beg + a.seg_rows < p.n ? r_beg + a.seg_rows : p.n;
    if (r_beg >= p.n) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = vsl * L::cols, vw = wave * 16;  // first column of the workgroup, of the wave inside it
    const int l16 = lane & 15, g = lane >> 4;

    // The state slice of this wave: tile dt holds d = 16 dt + 4 g + i, v = v0 + vw + l16
    f4 s[KD / 16];
    const int64_t state_elems = (int64_t)a.dp * a.vp;
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * state_elems : nullptr;
    float *seg_state = a.segments > 1 ? a.ws + (((int64_t)b * a.heads + h) * a.segments + seg) * (state_elems + a.dp + 16) : nullptr;
    const float *from = STATES ? nullptr : (a.segments > 1 ? seg_state : (p.pos0 > 0 ? pool : nullptr));
    // (a state as a buffer: rows past dp lie past its end, columns past vp get an offset outside)
    const int state_bytes = (int)state_elems * 4, v = v0 + vw + l16;
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
    float decayed = 1.f;  // STATES: the segment's factor of channel tid

    const uint16_t *uq = reinterpret_cast<const uint16_t *>(a.q) + p.row0 * a.ldq + h * a.dim;
    const uint16_t *uz = reinterpret_cast<const uint16_t *>(a.z) + p.row0 * a.ldz + h * a.dim;
    const uint16_t *uv = reinterpret_cast<const uint16_t *>(a.v) + p.row0 * a.ldv + h * a.vdim + v0;
    const int vcols = a.vdim - v0 < L::cols ? a.vdim - v0 : L::cols;

    // A unit: channels 2 pair, 2 pair + 1 of rows 8 oct .. 8 oct + 7; lanes 0 .. 31 and 32 .. 63 of a wave share a block.
    int pair[L::passes], oct[L::passes];
    bool mine[L::passes];
    float bias[L::passes][2], lower[L::passes][2];
#pragma unroll
    for (int u = 0; u < L::passes; ++u) {
        const int group = wave + NW * u, per = kPairs / 32;
        mine[u] = group * 64 < L::units;
        pair[u] = 32 * (group % per) + (lane & 31);
        oct[u] = group / per * 2 + (lane >> 5);
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const int d = 2 * pair[u] + e, c = h * a.dim + d;
            bias[u][e] = d < a.dim && a.bias ? a.bias[c] : 0.f;
            lower[u][e] = d < a.dim ? a.lower[c] : 1.f;
        }
    }
    uint32_t zr[L::passes][8], qr[STATES ? 1 : L::passes][8];
    la_u2 vr[L::vLoads];
    auto fetch = [&](int r0) {
        const int nr = r_end - r0 < kRows ? r_end - r0 : kRows;
        const __amdgpu_buffer_rsrc_t tz = la_tile(uz + r0 * a.ldz, a.ldz, nr, a.dim), tv = la_tile(uv + r0 * a.ldv, a.ldv, nr, vcols);
        const __amdgpu_buffer_rsrc_t tq = la_tile(uq + r0 * a.ldq, a.ldq, nr, a.dim);
#pragma unroll
        for (int u = 0; u < L::passes; ++u) {
            if (!mine[u]) continue;
            const bool there = 2 * pair[u] < a.dim;
#pragma unroll
            for (int r = 0; r < 8; ++r) {
                zr[u][r] = __builtin_amdgcn_raw_buffer_load_b32(tz, there ? (uint32_t)((8 * oct[u] + r) * a.ldz + 2 * pair[u]) * 2u : kLaOutside, 0, 0);
                if constexpr (!STATES)
                    qr[u][r] = __builtin_amdgcn_raw_buffer_load_b32(tq, there ? (uint32_t)((8 * oct[u] + r) * a.ldq + 2 * pair[u]) * 2u : kLaOutside, 0, 0);
            }
        }
#pragma unroll
        for (int n = 0; n < L::vLoads; ++n) {
            const int c = tid + kThr * n, row = c / (L::cols / 4), col = c % (L::cols / 4) * 4;
            vr[n] = __builtin_amdgcn_raw_buffer_load_b64(tv, la_block_off(a.ldv, row, col, vcols), 0, 0);
        }
    };
    fetch(r_beg);
    for (int r0 = r_beg; r0 < r_end; r0 += kRows) {
        const int nv = r_end - r0 < kRows ? r_end - r0 : kRows;
        if (!STATES && tid < L::blocks) unsafe[tid] = 0;
        // ---- operands ----
        bool bad[L::passes];
#pragma unroll
        for (int u = 0; u < L::passes; ++u) {
            bad[u] = false;
            if (!mine[u]) continue;
            float f[8][2], k[8][2], up[2] = {1.f, 1.f};
#pragma unroll
            for (int r = 0; r < 8; ++r)
#pragma unroll
                for (int e = 0; e < 2; ++e) {
                    const float z = __builtin_bit_cast(float, e ? zr[u][r] & 0xffff0000u : zr[u][r] << 16) + bias[u][e];
                    cl_gate<pa_bf16>(z, lower[u][e], f[r][e], k[r][e]);
                    if (8 * oct[u] + r >= nv) {
                        f[r][e] = 1.f;
                        k[r][e] = 0.f;
                    }
                    up[e] *= f[r][e];
                }
            // the other half of the block: what lies ahead of this one, and behind it
            const bool second = lane >= 32;
            float ahead[2], behind[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const float other = __shfl_xor(up[e], 32, 64);
                ahead[e] = second ? other : 1.f;
                behind[e] = second ? 1.f : other;
                if (second) whole[(oct[u] >> 1) * KD + 2 * pair[u] + e] = up[e] * other;
                bad[u] = bad[u] || up[e] * other < kClSmall;
            }
            uint32_t *dst = reinterpret_cast<uint32_t *>(k_hi) + (8 * oct[u] * kPitch) / 2 + pair[u];
            constexpr int kRow = kPitch / 2, kTerm = L::elems / 2;
            {
                float back[2] = {behind[0], behind[1]};
#pragma unroll
                for (int r = 7; r >= 0; --r) {
                    uint32_t hi, lo;
                    la_split2(k[r][0] * back[0], k[r][1] * back[1], hi, lo);
                    dst[r * kRow] = hi;
                    dst[kTerm + r * kRow] = lo;
                    back[0] *= f[r][0];
                    back[1] *= f[r][1];
                }
            }
            if constexpr (!STATES) {
                float fwd[2] = {ahead[0], ahead[1]};
#pragma unroll
                for (int r = 0; r < 8; ++r) {
                    float q[2], inv[2];
#pragma unroll
                    for (int e = 0; e < 2; ++e) {
                        fwd[e] *= f[r][e];
                        q[e] = __builtin_bit_cast(float, e ? qr[u][r] & 0xffff0000u : qr[u][r] << 16);
                        if (a.silu) q[e] = row_silu<pa_bf16>(q[e]);
                        q[e] *= fwd[e];
                        inv[e] = k[r][e] * __builtin_amdgcn_rcpf(fwd[e]);
                    }
                    uint32_t hi, lo;
                    la_split2(q[0], q[1], hi, lo);
                    dst[2 * kTerm + r * kRow] = hi;
                    dst[3 * kTerm + r * kRow] = lo;
                    la_split2(inv[0], inv[1], hi, lo);
                    dst[4 * kTerm + r * kRow] = hi;
                    dst[5 * kTerm + r * kRow] = lo;
                }
            }
        }
#pragma unroll
        for (int n = 0; n < L::vLoads; ++n) {
            const int c = tid + kThr * n, row = c / (L::cols / 4), col = c % (L::cols / 4) * 4;
            *reinterpret_cast<la_u2 *>(v_s + row * L::vPitch + col) = vr[n];
        }
        if (r0 + kRows < r_end) fetch(r0 + kRows);
        __syncthreads();
        if constexpr (!STATES) {
            // (flags go up behind the barrier that follows their clearing, and are read behind the next)
#pragma unroll
            for (int u = 0; u < L::passes; ++u)
                if (bad[u]) unsafe[oct[u] >> 1] = 1;
            __syncthreads();
            // ---- scores: keys 4 g + i, row l16 of the wave's block ----
            if (wave < L::blocks) {
                const int first = wave * kClBlock;
                f4 sc = f4{0.f, 0.f, 0.f, 0.f};
                if (unsafe[wave] == 0) {
#pragma unroll
                    for (int kk = 0; kk < KD / 32; ++kk) {
                        const int at = (first + l16) * kPitch + 32 * kk + 8 * g;
                        const bf8 kh = la_read8(i_hi + at), kl = la_read8(i_lo + at), qh = la_read8(q_hi + at), ql = la_read8(q_lo + at);
                        sc = la_mfma(kl, qh, sc);
                        sc = la_mfma(kh, ql, sc);
                        sc = la_mfma(kh, qh, sc);
                    }
                } else {
                    const int n = nv - first;
                    sc = cl_slow_scores<KD>(uq + (r0 + first) * a.ldq, a.ldq, uz + (r0 + first) * a.ldz, a.ldz, a.bias ? a.bias + h * a.dim : nullptr,
                                            a.lower + h * a.dim, a.dim, a.silu, n < 0 ? 0 : n > kClBlock ? kClBlock : n,
                                            reinterpret_cast<float *>(i_hi + first * kPitch), reinterpret_cast<float *>(i_lo + first * kPitch));
                }
#pragma unroll
                for (int i = 0; i < 4; ++i) sc[i] = 4 * g + i <= l16 ? sc[i] : 0.f;
                uint4 x;
                la_split2(sc[0], sc[1], x.x, x.z);
                la_split2(sc[2], sc[3], x.y, x.w);
                scores[wave * 64 + lane] = x;
            }
            __syncthreads();
        }
        // ---- blocks in turn; every wave its own columns ----
#pragma unroll 1
        for (int blk = 0; blk < L::blocks; ++blk) {
            if (blk * kClBlock >= nv) break;
            const int first = blk * kClBlock;
            // V^T or V: rows 4 g .. 4 g + 3 of the block, column l16 of the wave, once for each term beside it
            const la_bf4 v4 = la_read_tr(v_s + (first + 4 * g + (l16 >> 2)) * L::vPitch + vw + 4 * (l16 & 3));
            const bf8 v8 = la_join(v4, v4);
            if constexpr (!STATES) {
                f4 o = f4{0.f, 0.f, 0.f, 0.f};  // v = 4 g + i of the wave's columns, t = l16
#pragma unroll
                for (int dd = 0; dd < KD / 32; ++dd) {
                    LaSplit sp;
#pragma unroll
                    for (int j = 0; j < 4; ++j)
                        la_split2(s[2 * dd + j / 2][2 * j % 4], s[2 * dd + j / 2][2 * j % 4 + 1], sp.hi[j], sp.lo[j]);
                    const bf8 hi = sp.high(), lo = sp.low();
                    const int at = (first + l16) * kPitch + 32 * dd + 4 * g;
                    const bf8 qh = la_read44(q_hi + at, q_hi + at + 16), ql = la_read44(q_lo + at, q_lo + at + 16);
                    o = la_mfma(lo, qh, o);
                    o = la_mfma(hi, ql, o);
                    o = la_mfma(hi, qh, o);
                }
                o = la_mfma(v8, __builtin_bit_cast(bf8, scores[blk * 64 + lane]), o);
                const int ldo = a.heads * a.vdim, c = vw + 4 * g;
                const uint16_t *out = reinterpret_cast<const uint16_t *>(a.out) + (p.row0 + r0 + first) * (int64_t)ldo + h * a.vdim + v0;
                const int n = nv - first < kClBlock ? nv - first : kClBlock;
                const __amdgpu_buffer_rsrc_t dst = la_tile(out, ldo, n, vcols);
                const la_u2 x = {row_pack_bf16(o[0], o[1]), row_pack_bf16(o[2], o[3])};
                __builtin_amdgcn_raw_buffer_store_b64(x, dst, c < vcols ? (uint32_t)(l16 * ldo + c) * 2u : kLaOutside, 0, 0);
            }
            const float *keep = whole + blk * KD + 4 * g;
            const __bf16 *kh = k_hi + (first + 4 * g + (l16 >> 2)) * kPitch + 4 * (l16 & 3), *kl = kh + L::elems;
#pragma unroll
            for (int dt = 0; dt < KD / 16; ++dt) {
                const f4 f = *reinterpret_cast<const f4 *>(keep + 16 * dt);
#pragma unroll
                for (int i = 0; i < 4; ++i) s[dt][i] *= f[i];
                s[dt] = la_mfma(la_join(la_read_tr(kh + 16 * dt), la_read_tr(kl + 16 * dt)), v8, s[dt]);
            }
        }
        if (STATES && tid < KD)
            for (int blk = 0; blk < L::blocks; ++blk) decayed *= whole[blk * KD + tid];
        __syncthreads();  // the next rows' operands may be written now
    }
    float *to = STATES ? seg_state : (a.segments > 1 ? nullptr : pool);
    if (!to) return;
    const __amdgpu_buffer_rsrc_t dst = __builtin_amdgcn_make_buffer_rsrc((void *)to, 0, state_bytes, 0x00020000);
#pragma unroll
    for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float x = s[dt][i];
            __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(uint32_t, x), dst, soff + (16 * dt + i) * a.vp * 4, 0, 0);
        }
    if (STATES && vsl == 0 && tid < KD && tid < a.dp) to[state_elems + tid] = decayed;  // (every value slice has the same)
}

// Segment contributions -> start states, in place; the state after the last segment goes back to the pool.
__global__ __launch_bounds__(256) void channel_scan_kernel(const ClArgs a) {
    const int h = blockIdx.y, b = blockIdx.z;
    ClPortion p;
    if (!cl_portion(a, b, p)) return;
    const int64_t n4 = (int64_t)a.dp * a.vp / 4, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n4) return;
    const int d = (int)(i * 4 / a.vp);
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * 4 * n4 : nullptr;
    const int64_t stride = 4 * n4 + a.dp + 16;
    float *seg = a.ws + ((int64_t)b * a.heads + h) * a.segments * stride;
    float4 cur = pool && p.pos0 > 0 ? reinterpret_cast<const float4 *>(pool)[i] : make_float4(0.f, 0.f, 0.f, 0.f);
    for (int j = 0; (int64_t)j * a.seg_rows < p.n; ++j, seg += stride) {
        const float keep = seg[4 * n4 + d];
        float4 *at = reinterpret_cast<float4 *>(seg) + i;
        const float4 add = *at;
        *at = cur;
        cur = make_float4(fmaf(keep, cur.x, add.x), fmaf(keep, cur.y, add.y), fmaf(keep, cur.z, add.z), fmaf(keep, cur.w, add.w));
    }
    if (pool) reinterpret_cast<float4 *>(pool)[i] = cur;
}

template <int KD, int NW> int launch_chunks(const ClArgs &a, int batch, hipStream_t s) {
    constexpr size_t lds = ClTile<KD, NW, false>::bytes, lds_states = ClTile<KD, NW, true>::bytes;
    static_assert(lds <= 160 * 1024 && lds_states <= 160 * 1024, "LDS of one compute unit");
    const int slices = (a.vdim + 16 * NW - 1) / (16 * NW);
    const dim3 grid((unsigned)a.heads, (unsigned)(slices * a.segments), (unsigned)batch), block(64 * NW);
    if (a.segments > 1) {
        if (int rc = la_big_lds(channel_chunk_kernel<KD, NW, true>, lds_states, "pa_channel_linear")) return rc;
        channel_chunk_kernel<KD, NW, true><<<grid, block, lds_states, s>>>(a);
        const unsigned gx = (unsigned)(((int64_t)a.dp * a.vp / 4 + 255) / 256);
        channel_scan_kernel<<<dim3(gx, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s>>>(a);
    }
    if (int rc = la_big_lds(channel_chunk_kernel<KD, NW, false>, lds, "pa_channel_linear")) return rc;
    channel_chunk_kernel<KD, NW, false><<<grid, block, lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_channel_linear (chunks)");
    return PA_OK;
}

template <typename T> void launch_recurrent(const ClArgs &a, int batch, hipStream_t s) {
    // (a head's slices, whose rows lie side by side in memory, run at the same time)
    const dim3 grid((unsigned)((a.vdim + kClCols - 1) / kClCols), (unsigned)a.heads, (unsigned)batch), block(256);
    if (a.dim <= 64) channel_recurrent_kernel<T, 4><<<grid, block, 0, s>>>(a);
    else if (a.dim <= 128) channel_recurrent_kernel<T, 8><<<grid, block, 0, s>>>(a);
    else channel_recurrent_kernel<T, 16><<<grid, block, 0, s>>>(a);
}

int cl_plan(int64_t batch, int heads, int vdim, int max_q_len) {
    const int cols = la_value_cols(vdim);
    return la_segments(batch * heads * ((vdim + cols - 1) / cols), la_cus(), max_q_len);
}

}  // namespace

extern "C" size_t pa_channel_linear_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len) {
    pa_clear_error();
    if (batch < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || max_q_len < 0) {
        pa_fail(PA_ERR_INVALID_ARG, "pa_channel_linear_workspace_bytes: sizes out of range");
        return 0;
    }
    return gl_workspace_bytes(batch, num_heads, dim, vdim, cl_plan(batch, num_heads, vdim, max_q_len));
}

extern "C" int pa_channel_linear(const void *q, int64_t q_stride, int q_act, const void *forget, int64_t f_stride, const float *f_bias,
                                 const float *lower, const void *v, int64_t v_stride, int64_t n_rows, float *state, int64_t state_rows,
                                 const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts, const int32_t *state_slots,
                                 int batch, int max_q_len, void *out, int num_heads, int dim, int vdim, int dtype, void *workspace,
                                 size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && state_rows >= 0 && max_q_len >= 0, "pa_channel_linear: a count is negative");
    PA_REQUIRE(num_heads > 0 && dim > 0 && vdim > 0, "pa_channel_linear: heads / dim / vdim must be positive");
    PA_REQUIRE(num_heads <= 65535 && batch <= 65535, "pa_channel_linear: heads=%d / batch=%d above 65535", num_heads, batch);
    PA_REQUIRE(q_act == PA_ACT_NONE || q_act == PA_ACT_SILU, "q_act=%d is unknown", q_act);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_channel_linear: dtype=%d is not F32 or BF16", dtype);
    if (dim > 256) return pa_fail(PA_ERR_UNSUPPORTED, "pa_channel_linear: dim=%d above 256", dim);
    PA_REQUIRE(q_stride >= (int64_t)num_heads * dim && f_stride >= (int64_t)num_heads * dim && v_stride >= (int64_t)num_heads * vdim,
               "pa_channel_linear: a stride is shorter than its row");
    PA_REQUIRE((int64_t)num_heads * (dim + vdim) <= 0x7fffffff, "pa_channel_linear: rows are too long");
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "pa_channel_linear: q_lens and q_starts come together");
    if (n_rows == 0 || batch == 0 || (q_lens && max_q_len == 0)) return PA_OK;
    PA_REQUIRE(q && forget && lower && v && state && ctx_lens && state_slots && out, "pa_channel_linear: NULL argument");
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    PA_REQUIRE(pa_aligned16(state), "pa_channel_linear: the state must be 16-byte aligned");
    ClArgs a{};
    a.q = q; a.z = forget; a.v = v; a.ldq = q_stride; a.ldz = f_stride; a.ldv = v_stride; a.bias = f_bias; a.lower = lower;
    a.silu = q_act == PA_ACT_SILU; a.n_rows = n_rows; a.state = state; a.state_rows = state_rows; a.ctx_lens = ctx_lens;
    a.q_lens = q_lens; a.q_starts = q_starts; a.state_slots = state_slots; a.out = out; a.heads = num_heads; a.dim = dim;
    a.vdim = vdim; a.dp = la_pad16(dim); a.vp = la_pad16(vdim); a.segments = 1;
    hipStream_t s = (hipStream_t)stream;
    // single rows, 32-bit rows, rows that are not whole 8-byte vectors, rows too far apart for 32-bit offsets
    const uintptr_t at = (uintptr_t)q | (uintptr_t)forget | (uintptr_t)v | (uintptr_t)out;
    const int64_t most = 1 << 22;
    if (!q_lens || dtype == PA_F32 || dim % 4 != 0 || vdim % 4 != 0 || q_stride % 4 != 0 || f_stride % 4 != 0 || v_stride % 4 != 0 ||
        (at & 7u) != 0 || q_stride > most || f_stride > most || v_stride > most || (int64_t)num_heads * vdim > most) {
        if (dtype == PA_F32) launch_recurrent<float>(a, batch, s);
        else launch_recurrent<pa_bf16>(a, batch, s);
        PA_CHECK_LAUNCH("pa_channel_linear");
        return PA_OK;
    }
    a.segments = cl_plan(batch, num_heads, vdim, max_q_len);
    while (a.segments > 1 && (!workspace || gl_workspace_bytes(batch, num_heads, dim, vdim, a.segments) > workspace_bytes))
        --a.segments;
    a.seg_rows = la_segment_rows(max_q_len, a.segments);
    a.ws = (float *)workspace;
    PA_REQUIRE(a.segments == 1 || pa_aligned16(workspace), "the workspace must be 16-byte aligned");
    const bool wide = la_value_cols(vdim) == 128;
    if (dim <= 64) return wide ? launch_chunks<64, 8>(a, batch, s) : launch_chunks<64, 4>(a, batch, s);
    if (dim <= 128) return wide ? launch_chunks<128, 8>(a, batch, s) : launch_chunks<128, 4>(a, batch, s);
    return wide ? launch_chunks<256, 8>(a, batch, s) : launch_chunks<256, 4>(a, batch, s);
}
