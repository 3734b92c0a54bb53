// Linear recurrences whose decay and input weight come with every token: per head S_t = a_t S_(t-1) + b_t k_t v_t^T and a
// read-out S_t^T q_t, with S in 32-bit floats, kept per sequence in a pool of state slots.  Two kinds:
//
//   kSsd    Mamba-2's state-space duality: a = exp(-A dt), b = dt = softplus(raw + bias); o = S^T q + D v.  Heads of a
//           group share q and k.
//   kMlstm  xLSTM's matrix memory: log gates i and f under a soft cap, a running maximum m (starting at 0) that both are
//           taken relative to, a normaliser n that follows k with the same factors; o = S^T q / (max(|n.q|, exp(-m)) + 1e-6).
//
// Two kernels, as for the constant decays of lightning.hip.  The recurrent one (a decode step, and 32-bit prompts) reads
// the state once, walks its rows token by token in registers and writes the state once.  The chunked one (16-bit
// prompts) multiplies 64 rows at a time on the matrix cores.  With F the running sum of log decays inside the chunk and
// M the running maximum of i - F (kSsd: i = 0 and M = 0; b stays a factor), both from one wave's prefix scans,
//     O = diag(e^(F_t or m0 - M_t)) Q S + ((Q K^T) * e^(F_t - F_s or i_s - F_s - M_t) b_s, s <= t) V
// and the state moves on by the same weights at the chunk's last row.  All logarithms are to base 2.
// n is followed by the vector units; its product with q and the sums of the weighted scores give the denominators.
#include "linear_tiles.h"

namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kGlNone = -1.0e30f;  // finite stand-in for minus infinity

enum { kSsd = PA_GL_SSD, kMlstm = PA_GL_MLSTM };

struct GlArgs {
    const void *q, *k, *v;  // row strides ldq, ldk, ldv; head h: q, k at h / per_group * dim, v at h * vdim
    int64_t ldq, ldk, ldv;
    const void *ga, *gb;    // gate logits [row][head] at stride ldg: kSsd ga = raw dt; kMlstm ga = i, gb = f
    int64_t ldg;
    const float *pa, *pb, *pc;  // [heads]: kSsd dt bias, A, D; kMlstm biases of i and f
    float cap, q_scale, den_eps;
    int64_t n_rows;
    float *state;  // [state_rows][heads][head_floats]: S [dp][vp], then per 64 value columns n [dp] and m (kMlstm)
    int64_t state_rows, head_floats;
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots;
    void *out;  // [rows][heads * vdim]
    float *ws;  // segment states: S [dp][vp], n [dp], m, log decay, starting m
    int heads, per_group, dim, vdim, dp, vp;
    int segments, seg_rows;
};

struct GlPortion {
    int n, pos0;
    int64_t row0, slot;
};
__device__ __forceinline__ bool gl_portion(const GlArgs &a, int b, GlPortion &p) {
    p.n = a.q_lens ? a.q_lens[b] : 1;
    p.row0 = a.q_starts ? a.q_starts[b] : b;
    p.pos0 = a.ctx_lens[b] - p.n;
    p.slot = a.state_slots[b];
    if (p.slot >= a.state_rows) p.slot = -1;
    return p.n > 0 && p.pos0 >= 0 && p.row0 >= 0 && p.row0 + p.n <= a.n_rows;
}

// ------------------------------------------------------------------ gates
__device__ __forceinline__ float gl_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

struct GlHead {  // a head's constants
    float a, b, c;
};
__device__ __forceinline__ GlHead gl_head(const GlArgs &a, int h) {
    return GlHead{a.pa[h], a.pb[h], a.pc ? a.pc[h] : 0.f};
}
// Log decay (base 2) and, kSsd, the input weight or, kMlstm, its logarithm (base 2).
template <int KIND> __device__ __forceinline__ void gl_gate(const GlArgs &a, const GlHead &hd, float ra, float rb, float &decay, float &in) {
    if constexpr (KIND == kSsd) {
        in = gl_softplus(ra + hd.a);
        decay = -hd.b * in * kLog2e;
    } else {
        in = a.cap * tanhf((ra + hd.a) / a.cap) * kLog2e;
        decay = -gl_softplus(-a.cap * tanhf((rb + hd.b) / a.cap)) * kLog2e;
    }
}

// ------------------------------------------------------------------ token by token
constexpr int kRecCols = 64;  // value columns per workgroup: 16 lanes x float4, 16 groups of lanes over the rows of S

// R: rows of S per thread (16 R >= dim).  kMlstm: thread d follows n[d].
template <typename T, int R, int KIND> __global__ __launch_bounds__(256, 4) void gated_recurrent_kernel(const GlArgs a) {
    __shared__ float qs[16 * R], ks[16 * R], vs[kRecCols];
    __shared__ float4 red[16][kRecCols / 4];
    __shared__ float redn[4];
    const int h = blockIdx.y, b = blockIdx.z, v0 = blockIdx.x * kRecCols;
    GlPortion p;
    if (!gl_portion(a, b, p)) return;
    const int tid = threadIdx.x, col = tid % 16 * 4, grp = tid / 16;
    const bool live = v0 + col < a.vp;  // (vp is a multiple of 16)
    float *head = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * a.head_floats : nullptr;
    float *sp = head ? head + v0 + col : nullptr;
    float *np = head ? head + (int64_t)a.dp * a.vp + blockIdx.x * (int64_t)(a.dp + 16) : nullptr;  // this workgroup's copy
    const bool resume = head && p.pos0 > 0;
    float4 s[R];
    float n = 0.f, m = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        s[r] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (resume && live && d < a.dp) s[r] = *reinterpret_cast<const float4 *>(sp + (int64_t)d * a.vp);
    }
    if (KIND == kMlstm && resume) {
        if (tid < a.dp && tid < 16 * R) n = np[tid];
        m = np[a.dp];
    }
    const GlHead hd = gl_head(a, h);
    const int g = h / a.per_group;
    const T *q = reinterpret_cast<const T *>(a.q) + g * a.dim, *k = reinterpret_cast<const T *>(a.k) + g * a.dim;
    const T *v = reinterpret_cast<const T *>(a.v) + h * a.vdim + v0;
    for (int t = 0; t < p.n; ++t) {
        const int64_t row = p.row0 + t;
        for (int i = tid; i < 2 * 16 * R + kRecCols; i += 256) {
            if (i < 16 * R) {
                qs[i] = i < a.dim ? pa_scalar<T>::load(q + row * a.ldq + i) : 0.f;
            } else if (i < 32 * R) {
                const int d = i - 16 * R;
                ks[d] = d < a.dim ? pa_scalar<T>::load(k + row * a.ldk + d) : 0.f;
            } else {
                const int c = i - 32 * R;
                vs[c] = v0 + c < a.vdim ? pa_scalar<T>::load(v + row * a.ldv + c) : 0.f;
            }
        }
        const float ra = pa_scalar<T>::load(reinterpret_cast<const T *>(a.ga) + row * a.ldg + h);
        const float rb = KIND == kMlstm ? pa_scalar<T>::load(reinterpret_cast<const T *>(a.gb) + row * a.ldg + h) : 0.f;
        float keep, in;
        gl_gate<KIND>(a, hd, ra, rb, keep, in);
        if (KIND == kMlstm) {
            const float next = fmaxf(keep + m, in);
            keep = exp2f(keep + m - next);
            in = exp2f(in - next);
            m = next;
        } else {
            keep = exp2f(keep);
        }
        __syncthreads();
        float4 x = *reinterpret_cast<const float4 *>(vs + col);
        x = make_float4(in * x.x, in * x.y, in * x.z, in * x.w);
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float kd = ks[grp + 16 * r], qd = qs[grp + 16 * r];
            s[r].x = fmaf(keep, s[r].x, kd * x.x); s[r].y = fmaf(keep, s[r].y, kd * x.y);
            s[r].z = fmaf(keep, s[r].z, kd * x.z); s[r].w = fmaf(keep, s[r].w, kd * x.w);
            o.x = fmaf(qd, s[r].x, o.x); o.y = fmaf(qd, s[r].y, o.y);
            o.z = fmaf(qd, s[r].z, o.z); o.w = fmaf(qd, s[r].w, o.w);
        }
        red[grp][tid % 16] = o;
        if (KIND == kMlstm) {
            float nq = 0.f;
            if (tid < 16 * R) {
                n = fmaf(keep, n, in * ks[tid]);
                nq = qs[tid] * n;
            }
            nq = pa_group_sum<64>(nq);
            if (tid % 64 == 0) redn[tid / 64] = nq;
        }
        __syncthreads();
        if (tid < kRecCols && v0 + tid < a.vdim) {
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) sum += reinterpret_cast<const float *>(red[i])[tid];
            if (KIND == kMlstm) {
                const float den = (redn[0] + redn[1]) + (redn[2] + redn[3]);
                sum = a.q_scale * sum / (fmaxf(fabsf(a.q_scale * den), exp2f(-m)) + a.den_eps);
            } else {
                sum = fmaf(hd.c, vs[tid], sum);
            }
            pa_scalar<T>::store(reinterpret_cast<T *>(a.out) + row * ((int64_t)a.heads * a.vdim) + h * a.vdim + v0 + tid, sum);
        }
        if (KIND == kSsd) __syncthreads();  // (vs is read above)
        // (otherwise: the next token's writes to qs, ks, vs follow every thread's reads of them, before the barrier above;
        // its writes to red and redn come after its own barrier, which the threads that sum here reach afterwards)
    }
    if (!head) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        if (live && d < a.dp) *reinterpret_cast<float4 *>(sp + (int64_t)d * a.vp) = s[r];
    }
    if (KIND == kMlstm) {
        if (tid < a.dp && tid < 16 * R) np[tid] = n;
        if (tid == 0) np[a.dp] = m;
    }
}

// ------------------------------------------------------------------ chunks on the matrix cores
// Per-chunk vectors in LDS (64 rows each)
struct GlRows {
    float row[64], col[64], mul[64];  // a score (t, s) is weighted by 2^(row[t] + col[s]) mul[s]
    float inter[64], add[64];         // rows' factor on Q S; weights of the chunk's rows in the new state
    float low[64];                    // exp(-m)
    float whole, pad[15];             // factor on the old state
};

// Elements of the tiles: Q and K row-major, the two terms of the weighted scores, the transposed K and V.
template <int KD> constexpr int gl_r_elems() { return 64 * (KD + 8); }
constexpr int kGlAElems = 2 * 64 * kLaPitchA;
template <int KD, int NW> constexpr int gl_t_elems() { return (KD + 16 * NW) * 64; }
template <int KD, int NW, int KIND, bool STATES> constexpr size_t gl_lds_bytes() {
    const size_t elems = STATES ? 2 * gl_t_elems<KD, NW>()  // (double-buffered: one barrier per chunk)
                                : 2 * gl_r_elems<KD>() + kGlAElems + gl_t_elems<KD, NW>();
    return elems * 2 + (STATES ? 2 : 1) * sizeof(GlRows) + (KIND == kMlstm && !STATES ? (3 * 64 + KD) * 4 : 0);
}

// Inclusive scans over the wave: rows of 16 lanes by shifts inside the row, then the rows before.
template <int CTRL> __device__ __forceinline__ float gl_shift(float x, float outside) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, outside), __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, false));
}
__device__ __forceinline__ float gl_lane(float x, int lane) {
    return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), lane));
}
__device__ __forceinline__ float gl_scan_add(float x, int lane) {
    x += gl_shift<0x111>(x, 0.f);
    x += gl_shift<0x112>(x, 0.f);
    x += gl_shift<0x114>(x, 0.f);
    x += gl_shift<0x118>(x, 0.f);
    const float r0 = gl_lane(x, 15), r1 = r0 + gl_lane(x, 31), r2 = r1 + gl_lane(x, 47);
    return x + (lane < 16 ? 0.f : lane < 32 ? r0 : lane < 48 ? r1 : r2);
}
__device__ __forceinline__ float gl_scan_max(float x, int lane) {
    x = fmaxf(x, gl_shift<0x111>(x, kGlNone));
    x = fmaxf(x, gl_shift<0x112>(x, kGlNone));
    x = fmaxf(x, gl_shift<0x114>(x, kGlNone));
    x = fmaxf(x, gl_shift<0x118>(x, kGlNone));
    const float r0 = gl_lane(x, 15), r1 = fmaxf(r0, gl_lane(x, 31)), r2 = fmaxf(r1, gl_lane(x, 47));
    return fmaxf(x, lane < 16 ? kGlNone : lane < 32 ? r0 : lane < 48 ? r1 : r2);
}

// KD: dim padded to 64, 128 or 256.  NW: waves; each owns 16 value columns.  All products are taken transposed (value
// columns, or keys, as the rows of the result), so that a lane holds four consecutive elements of one row t.
// STATES: only the segment's own contribution to the state, to the workspace (first pass over a portion in segments).
template <int KD, int NW, int KIND, bool STATES>
__global__ __launch_bounds__(64 * NW, NW == 4 && KD == 256 ? 1 : 2) void gated_chunk_kernel(const GlArgs a) {
    constexpr int kCols = 16 * NW, kLdR = KD + 8, kThr = 64 * NW;
    constexpr int kDB = KD / 4, kKBlocks = 16 * kDB, kKPass = (kKBlocks + kThr - 1) / kThr;  // 4x4 blocks of K
    constexpr int kST = NW == 8 ? 2 : 4;  // score tiles per wave
    extern __shared__ __align__(16) char lds[];
    GlRows *rows = reinterpret_cast<GlRows *>(lds);
    float *nq_s = reinterpret_cast<float *>(rows + (STATES ? 2 : 1));  // kMlstm: n . q per row, two parts of the score sums, n
    float *sum_s = nq_s + 64, *n_s = sum_s + 128;
    __bf16 *tiles = reinterpret_cast<__bf16 *>(KIND == kMlstm && !STATES ? n_s + KD : nq_s);
    __bf16 *kt_s = tiles, *vt_s = kt_s + KD * 64;
    __bf16 *q_s = tiles + gl_t_elems<KD, NW>(), *k_s = q_s + gl_r_elems<KD>(), *a_hi = k_s + gl_r_elems<KD>();
    __bf16 *a_lo = a_hi + 64 * kLaPitchA;

    const int h = blockIdx.x, seg = blockIdx.y % a.segments, vsl = blockIdx.y / a.segments, b = blockIdx.z;
    GlPortion p;
    if (!gl_portion(a, b, p)) return;
    const int r_beg = seg * a.seg_rows, r_end = r_beg + a.seg_rows < p.n ? r_beg + a.seg_rows : p.n;
    if (r_beg >= p.n) return;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = vsl * kCols, vw = wave * 16;  // first column of the workgroup, of the wave inside it
    const int l16 = tid & 15, g = (tid & 63) >> 4;
    const GlHead hd = gl_head(a, h);

    // The state slice of this wave: tile dt holds d = 16 dt + 4 g + i, v = v0 + vw + l16
    f4 s[KD / 16];
    const int64_t state_elems = (int64_t)a.dp * a.vp;
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * a.head_floats : nullptr;
    float *seg_state = a.segments > 1 ? a.ws + (((int64_t)b * a.heads + h) * a.segments + seg) * (state_elems + a.dp + 16) : nullptr;
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
    // n and m of the workgroup: thread d follows n[d], the first wave m
    const int rep0 = v0 / kRecCols;
    float n_own = 0.f, m_prev = STATES ? kGlNone : 0.f, decayed = 0.f;
    if constexpr (KIND == kMlstm && !STATES) {
        const float *np = from ? from + state_elems + (a.segments > 1 ? 0 : rep0 * (a.dp + 16)) : nullptr;
        if (np) {
            if (tid < a.dp && tid < KD) n_own = np[tid];
            m_prev = a.segments > 1 ? np[a.dp + 2] : np[a.dp];
        }
        if (tid < KD) n_s[tid] = n_own;
    }

    const int grp = h / a.per_group;
    const uint16_t *uq = reinterpret_cast<const uint16_t *>(a.q) + p.row0 * a.ldq + grp * a.dim;
    const uint16_t *uk = reinterpret_cast<const uint16_t *>(a.k) + p.row0 * a.ldk + grp * a.dim;
    const uint16_t *uv = reinterpret_cast<const uint16_t *>(a.v) + p.row0 * a.ldv + h * a.vdim + v0;
    const pa_bf16 *ga = reinterpret_cast<const pa_bf16 *>(a.ga) + p.row0 * a.ldg + h;
    const pa_bf16 *gb = reinterpret_cast<const pa_bf16 *>(a.gb) + p.row0 * a.ldg + h;
    const int vcols = a.vdim - v0 < kCols ? a.vdim - v0 : kCols;
    LaBlock kb[kKPass], qb[STATES ? 1 : kKPass], vb;
    const uint32_t voff = la_block_off(a.ldv, tid / (kCols / 4) * 4, tid % (kCols / 4) * 4, vcols);
    float raw_a = 0.f, raw_b = 0.f;
    auto fetch = [&](int r0) {
        const int nr = r_end - r0 < kLaChunk ? r_end - r0 : kLaChunk;
        const __amdgpu_buffer_rsrc_t tk = la_tile(uk + r0 * a.ldk, a.ldk, nr, a.dim), tv = la_tile(uv + r0 * a.ldv, a.ldv, nr, vcols);
        if (wave == 0 && tid < nr) {
            raw_a = pa_scalar<pa_bf16>::load(ga + (r0 + tid) * a.ldg);
            if (KIND == kMlstm) raw_b = pa_scalar<pa_bf16>::load(gb + (r0 + tid) * a.ldg);
        }
        if (!STATES) {
            const __amdgpu_buffer_rsrc_t tq = la_tile(uq + r0 * a.ldq, a.ldq, nr, a.dim);
#pragma unroll
            for (int i = 0; i < kKPass; ++i) {
                const int blk = tid + kThr * i;
                qb[i] = la_load_block(tq, blk < kKBlocks ? la_block_off(a.ldq, blk / kDB * 4, blk % kDB * 4, a.dim) : kLaOutside,
                                      (uint32_t)a.ldq * 2u);
            }
        }
#pragma unroll
        for (int i = 0; i < kKPass; ++i) {
            const int blk = tid + kThr * i;
            kb[i] = la_load_block(tk, blk < kKBlocks ? la_block_off(a.ldk, blk / kDB * 4, blk % kDB * 4, a.dim) : kLaOutside,
                                  (uint32_t)a.ldk * 2u);
        }
        vb = la_load_block(tv, voff, (uint32_t)a.ldv * 2u);
    };
    fetch(r_beg);
    for (int r0 = r_beg; r0 < r_end; r0 += kLaChunk) {
        const int nv = r_end - r0 < kLaChunk ? r_end - r0 : kLaChunk;
#pragma unroll
        for (int i = 0; i < kKPass; ++i) {
            const int blk = tid + kThr * i, c = blk % kDB * 4, sr = blk / kDB * 4;
            if (kKBlocks % kThr != 0 && blk >= kKBlocks) continue;
            la_put_block<false>(kb[i], sr, c, STATES ? nullptr : k_s, kLdR, kt_s);
            if (!STATES) la_put_block<false>(qb[i], sr, c, q_s, kLdR, nullptr);
        }
        la_put_block<false>(vb, tid / (kCols / 4) * 4, tid % (kCols / 4) * 4, nullptr, 0, vt_s);
        if (wave == 0) {  // the chunk's gates, one row per lane
            float decay, in;
            gl_gate<KIND>(a, hd, raw_a, raw_b, decay, in);
            if (tid >= nv) decay = 0.f;
            const float f = gl_scan_add(decay, tid), f_last = gl_lane(f, 63);
            if constexpr (KIND == kSsd) {
                const float mul = tid < nv ? in : 0.f;
                rows->row[tid] = f;
                rows->col[tid] = -f;
                rows->mul[tid] = mul;
                rows->inter[tid] = exp2f(f);
                rows->add[tid] = exp2f(f_last - f) * mul;
                if (tid == 0) rows->whole = exp2f(f_last);
            } else {
                const float col = tid < nv ? in - f : kGlNone;
                const float top = fmaxf(m_prev, gl_scan_max(col, tid)), top_last = gl_lane(top, 63);
                rows->row[tid] = -top;
                rows->col[tid] = col;
                rows->inter[tid] = exp2f(m_prev - top);
                rows->add[tid] = exp2f(col - top_last);
                rows->low[tid] = exp2f(-(f + top));
                if (tid == 0) rows->whole = exp2f(m_prev - top_last);
                m_prev = f_last + top_last;
            }
            decayed += f_last;
        }
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
            // the rows' part from before the chunk: Q S, then its factors
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
            for (int tt = 0; tt < 4; ++tt) {
                const float f = rows->inter[16 * tt + l16];
#pragma unroll
                for (int i = 0; i < 4; ++i) o[tt][i] *= f;
            }
            if constexpr (KIND == kMlstm) {  // n . q: NW lanes per row
                const int t = tid / NW;
                constexpr int kPer = KD / NW;
                const __bf16 *qr = q_s + t * kLdR + tid % NW * kPer;
                const float *nr = n_s + tid % NW * kPer;
                float acc = 0.f;
#pragma unroll
                for (int d = 0; d < kPer; d += 8) {
                    const bf8 x = la_read8(qr + d);
#pragma unroll
                    for (int j = 0; j < 8; ++j) acc = fmaf((float)x[j], nr[d + j], acc);
                }
                acc = pa_group_sum<NW>(acc);
                if (tid % NW == 0) nq_s[t] = acc;
            }
            // the scores' weights
            const int t = 16 * rt + l16;
            const float row_w = rows->row[t];
            float sum = 0.f;
#pragma unroll
            for (int m = 0; m < kST; ++m) {
                const int st = NW == 8 ? 2 * m + (wave & 1) : m;
                if (st > rt + 1) continue;  // (tile rt + 1 is read as zeros when the last k-step covers it)
                const int c = 16 * st + 4 * g;
                const f4 cw = *reinterpret_cast<const f4 *>(rows->col + c);
                f4 x;
#pragma unroll
                for (int i = 0; i < 4; ++i) x[i] = c + i <= t ? sc[m][i] * __builtin_amdgcn_exp2f(row_w + cw[i]) : 0.f;
                if constexpr (KIND == kSsd) {
                    const f4 mul = *reinterpret_cast<const f4 *>(rows->mul + c);
#pragma unroll
                    for (int i = 0; i < 4; ++i) x[i] = fmaf(x[i], mul[i], c + i == t ? hd.c : 0.f);
                } else {
                    sum += (x[0] + x[1]) + (x[2] + x[3]);
                }
                uint2 hi, lo;
                la_split2(x[0], x[1], hi.x, lo.x);
                la_split2(x[2], x[3], hi.y, lo.y);
                *reinterpret_cast<uint2 *>(a_hi + t * kLaPitchA + c) = hi;
                *reinterpret_cast<uint2 *>(a_lo + t * kLaPitchA + c) = lo;
            }
            if constexpr (KIND == kMlstm) {
                sum += __shfl_xor(sum, 16, 64);
                sum += __shfl_xor(sum, 32, 64);
                if (g == 0) sum_s[(NW == 8 ? wave & 1 : 0) * 64 + t] = sum;
                if (NW == 4 && g == 1) sum_s[64 + t] = 0.f;
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
            const int ldo = a.heads * a.vdim;
            const uint16_t *first = reinterpret_cast<const uint16_t *>(a.out) + (p.row0 + r0) * (int64_t)ldo + h * a.vdim + v0;
            const __amdgpu_buffer_rsrc_t dst = la_tile(first, ldo, nv, vcols);
            const int c = vw + 4 * g;
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) {
                const int row = 16 * tt + l16;
                float f = a.q_scale;
                if constexpr (KIND == kMlstm) {
                    const float den = fmaf(rows->inter[row], nq_s[row], sum_s[row] + sum_s[64 + row]);
                    f /= fmaxf(fabsf(f * den), rows->low[row]) + a.den_eps;
                }
                const la_u2 x = {row_pack_bf16(o[tt][0] * f, o[tt][1] * f), row_pack_bf16(o[tt][2] * f, o[tt][3] * f)};
                __builtin_amdgcn_raw_buffer_store_b64(x, dst, c < vcols ? (uint32_t)(row * ldo + c) * 2u : kLaOutside, 0, 0);
            }
        }
        // S <- whole S + K^T (weights V)
        const float whole = rows->whole;
#pragma unroll
        for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i) s[dt][i] *= whole;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            LaSplit sp;
            const la_u4 bv = *reinterpret_cast<const la_u4 *>(vt_s + la_tr(vw + l16, 32 * kk + 8 * g));
            const f4 w0 = *reinterpret_cast<const f4 *>(rows->add + 32 * kk + 8 * g);
            const f4 w1 = *reinterpret_cast<const f4 *>(rows->add + 32 * kk + 8 * g + 4);
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
        if (KIND == kMlstm && tid < KD) {  // n likewise, with k alone
            float acc = whole * n_own;
#pragma unroll
            for (int c = 0; c < 8; ++c) {
                const bf8 x = la_read8(kt_s + la_tr(tid, 8 * c));
#pragma unroll
                for (int j = 0; j < 8; ++j) acc = fmaf(rows->add[8 * c + j], (float)x[j], acc);
            }
            n_own = acc;
            if (!STATES) n_s[tid] = acc;  // (read again after the next chunk's first barrier)
        }
        if constexpr (!STATES) {
            __syncthreads();  // the next chunk's tiles and gates may be written now
        } else {              // the other half of the tiles and gates
            kt_s = kt_s == tiles ? tiles + gl_t_elems<KD, NW>() : tiles;
            vt_s = kt_s + KD * 64;
            rows = rows == reinterpret_cast<GlRows *>(lds) ? rows + 1 : reinterpret_cast<GlRows *>(lds);
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
    if constexpr (STATES) {  // (every value slice has the same n, m and decay)
        if (vsl != 0) return;
        if (KIND == kMlstm && tid < a.dp && tid < KD) to[state_elems + tid] = n_own;
        if (tid == 0) {
            to[state_elems + a.dp] = m_prev;
            to[state_elems + a.dp + 1] = decayed;
        }
    } else if constexpr (KIND == kMlstm) {  // the copies of this workgroup's columns
        const int reps = (a.vdim + kRecCols - 1) / kRecCols;
        for (int r = rep0; r < reps && r < rep0 + (kCols + kRecCols - 1) / kRecCols; ++r) {
            float *np = to + state_elems + r * (a.dp + 16);
            if (tid < a.dp && tid < KD) np[tid] = n_own;
            if (tid == 0) np[a.dp] = m_prev;
        }
    }
}

// Segment contributions -> start states, in place; the state after the last segment goes back to the pool.  One thread per
// four elements of S, then of n; the first of n's threads also writes m.
template <int KIND> __global__ __launch_bounds__(256) void gated_scan_kernel(const GlArgs a) {
    const int h = blockIdx.y, b = blockIdx.z;
    GlPortion p;
    if (!gl_portion(a, b, p)) return;
    const int64_t n4 = (int64_t)a.dp * a.vp / 4, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const bool of_n = i >= n4;
    if (i >= n4 + (KIND == kMlstm ? a.dp / 4 : 0)) return;
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * a.head_floats : nullptr;
    const int64_t stride = 4 * n4 + a.dp + 16;
    float *seg = a.ws + ((int64_t)b * a.heads + h) * a.segments * stride;
    const bool resume = pool && p.pos0 > 0;
    float4 cur = resume ? reinterpret_cast<const float4 *>(pool)[i] : make_float4(0.f, 0.f, 0.f, 0.f);
    float m = KIND == kMlstm && resume ? pool[4 * n4 + a.dp] : 0.f;
    for (int j = 0; (int64_t)j * a.seg_rows < p.n; ++j, seg += stride) {
        const float decay = seg[4 * n4 + a.dp + 1];
        float keep, take = 1.f, next = 0.f;
        if (KIND == kMlstm) {
            const float m_seg = seg[4 * n4 + a.dp];
            next = fmaxf(decay + m, m_seg);
            keep = exp2f(decay + m - next);
            take = exp2f(m_seg - next);
        } else {
            keep = exp2f(decay);
        }
        float4 *at = reinterpret_cast<float4 *>(seg) + i;
        const float4 add = *at;
        *at = cur;
        if (KIND == kMlstm && i == n4) seg[4 * n4 + a.dp + 2] = m;
        cur = make_float4(fmaf(keep, cur.x, take * add.x), fmaf(keep, cur.y, take * add.y), fmaf(keep, cur.z, take * add.z),
                          fmaf(keep, cur.w, take * add.w));
        m = next;
    }
    if (!pool) return;
    if (!of_n) {
        reinterpret_cast<float4 *>(pool)[i] = cur;
        return;
    }
    const int reps = (a.vdim + kRecCols - 1) / kRecCols;
    for (int r = 0; r < reps; ++r) {
        float *np = pool + 4 * n4 + (int64_t)r * (a.dp + 16);
        reinterpret_cast<float4 *>(np)[i - n4] = cur;
        if (i == n4) np[a.dp] = m;
    }
}

template <int KD, int NW, int KIND> int launch_chunks(const GlArgs &a, int batch, hipStream_t s) {
    constexpr size_t lds = gl_lds_bytes<KD, NW, KIND, false>(), lds_states = gl_lds_bytes<KD, NW, KIND, true>();
    static_assert(lds <= 160 * 1024 && lds_states <= 160 * 1024, "LDS of one compute unit");
    const int slices = (a.vdim + 16 * NW - 1) / (16 * NW);
    const dim3 grid((unsigned)a.heads, (unsigned)(slices * a.segments), (unsigned)batch), block(64 * NW);
    if (a.segments > 1) {
        if (int rc = la_big_lds(gated_chunk_kernel<KD, NW, KIND, true>, lds_states, "pa_gated_linear")) return rc;
        gated_chunk_kernel<KD, NW, KIND, true><<<grid, block, lds_states, s>>>(a);
        const unsigned gx = (unsigned)(((int64_t)a.dp * a.vp / 4 + a.dp / 4 + 255) / 256);
        gated_scan_kernel<KIND><<<dim3(gx, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s>>>(a);
    }
    if (int rc = la_big_lds(gated_chunk_kernel<KD, NW, KIND, false>, lds, "pa_gated_linear")) return rc;
    gated_chunk_kernel<KD, NW, KIND, false><<<grid, block, lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_gated_linear (chunks)");
    return PA_OK;
}

template <int KIND> int launch_chunks_kind(const GlArgs &a, int batch, hipStream_t s) {
    const bool wide = la_value_cols(a.vdim) == 128;
    if (a.dim <= 64) return wide ? launch_chunks<64, 8, KIND>(a, batch, s) : launch_chunks<64, 4, KIND>(a, batch, s);
    if (a.dim <= 128) return wide ? launch_chunks<128, 8, KIND>(a, batch, s) : launch_chunks<128, 4, KIND>(a, batch, s);
    return wide ? launch_chunks<256, 8, KIND>(a, batch, s) : launch_chunks<256, 4, KIND>(a, batch, s);
}

template <typename T, int KIND> void launch_recurrent(const GlArgs &a, int batch, hipStream_t s) {
    // (a head's slices, whose rows lie side by side in memory, run at the same time)
    const dim3 grid((unsigned)((a.vdim + kRecCols - 1) / kRecCols), (unsigned)a.heads, (unsigned)batch), block(256);
    if (a.dim <= 64) gated_recurrent_kernel<T, 4, KIND><<<grid, block, 0, s>>>(a);
    else if (a.dim <= 128) gated_recurrent_kernel<T, 8, KIND><<<grid, block, 0, s>>>(a);
    else gated_recurrent_kernel<T, 16, KIND><<<grid, block, 0, s>>>(a);
}

int gl_plan(int64_t batch, int heads, int dim, int vdim, int max_q_len) {
    const int cols = la_value_cols(vdim);
    const int at_once = cols == 64 && dim <= 128 ? 2 * la_cus() : la_cus();  // workgroups: two of four waves fit a compute unit
    return la_segments(batch * heads * ((vdim + cols - 1) / cols), at_once, max_q_len);
}

}  // namespace

extern "C" size_t pa_gated_linear_state_floats(int kind, int dim, int vdim) {
    return (kind == kSsd || kind == kMlstm) && dim > 0 && vdim > 0 ? gl_state_floats(kind == kMlstm, dim, vdim) : 0;
}

extern "C" size_t pa_gated_linear_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len) {
    pa_clear_error();
    if (batch < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || max_q_len < 0) {
        pa_fail(PA_ERR_INVALID_ARG, "pa_gated_linear_workspace_bytes: sizes out of range");
        return 0;
    }
    return gl_workspace_bytes(batch, num_heads, dim, vdim, gl_plan(batch, num_heads, dim, vdim, max_q_len));
}

extern "C" int pa_gated_linear(int kind, const void *q, int64_t q_stride, const void *k, int64_t k_stride, const void *v,
                               int64_t v_stride, int heads_per_group, const void *gate_a, const void *gate_b,
                               int64_t gate_stride, const float *head_a, const float *head_b, const float *head_c, float cap,
                               float q_scale, float den_eps, int64_t n_rows, float *state, int64_t state_rows,
                               const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                               const int32_t *state_slots, int batch, int max_q_len, void *out, int num_heads, int dim,
                               int vdim, int dtype, void *workspace, size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(kind == kSsd || kind == kMlstm, "pa_gated_linear: kind=%d is unknown", kind);
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && state_rows >= 0 && max_q_len >= 0, "pa_gated_linear: a count is negative");
    PA_REQUIRE(num_heads > 0 && dim > 0 && vdim > 0, "pa_gated_linear: heads / dim / vdim must be positive");
    PA_REQUIRE(heads_per_group > 0 && num_heads % heads_per_group == 0, "heads_per_group=%d does not divide num_heads=%d",
               heads_per_group, num_heads);
    PA_REQUIRE(num_heads <= 65535 && batch <= 65535, "pa_gated_linear: heads=%d / batch=%d above 65535", num_heads, batch);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_gated_linear: dtype=%d is not F32 or BF16", dtype);
    if (dim > 256) return pa_fail(PA_ERR_UNSUPPORTED, "pa_gated_linear: dim=%d above 256", dim);
    const int groups = num_heads / heads_per_group;
    PA_REQUIRE(q_stride >= (int64_t)groups * dim && k_stride >= (int64_t)groups * dim && v_stride >= (int64_t)num_heads * vdim &&
                   gate_stride >= num_heads, "pa_gated_linear: a stride is shorter than its row");
    PA_REQUIRE((int64_t)num_heads * (dim + vdim) <= 0x7fffffff, "pa_gated_linear: rows are too long");
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "pa_gated_linear: q_lens and q_starts come together");
    PA_REQUIRE(kind == kSsd || cap > 0.f, "pa_gated_linear: cap must be positive");
    if (n_rows == 0 || batch == 0 || (q_lens && max_q_len == 0)) return PA_OK;
    PA_REQUIRE(q && k && v && gate_a && (gate_b || kind == kSsd) && head_a && head_b && (head_c || kind == kMlstm) && state &&
                   ctx_lens && state_slots && out, "pa_gated_linear: NULL argument");
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    PA_REQUIRE(pa_aligned16(state), "pa_gated_linear: the state must be 16-byte aligned");
    GlArgs a{};
    a.q = q; a.k = k; a.v = v; a.ldq = q_stride; a.ldk = k_stride; a.ldv = v_stride; a.per_group = heads_per_group;
    a.ga = gate_a; a.gb = kind == kSsd ? gate_a : gate_b; a.ldg = gate_stride; a.pa = head_a; a.pb = head_b; a.pc = head_c;
    a.cap = cap; a.q_scale = kind == kSsd ? 1.f : q_scale; a.den_eps = den_eps; a.n_rows = n_rows; a.state = state; a.state_rows = state_rows;
    a.ctx_lens = ctx_lens; a.q_lens = q_lens; a.q_starts = q_starts; a.state_slots = state_slots; a.out = out;
    a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.dp = la_pad16(dim); a.vp = la_pad16(vdim);
    a.head_floats = (int64_t)gl_state_floats(kind == kMlstm, dim, vdim);
    a.segments = 1;
    hipStream_t s = (hipStream_t)stream;
    // single rows, 32-bit rows, rows that are not whole 8-byte vectors, rows too far apart for 32-bit offsets
    const uintptr_t at = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)out;
    const int64_t most = 1 << 22;
    if (!q_lens || dtype == PA_F32 || dim % 4 != 0 || vdim % 4 != 0 || q_stride % 4 != 0 || k_stride % 4 != 0 ||
        v_stride % 4 != 0 || (at & 7u) != 0 || q_stride > most || k_stride > most || v_stride > most ||
        (int64_t)num_heads * vdim > most) {
        if (dtype == PA_F32) {
            if (kind == kSsd) launch_recurrent<float, kSsd>(a, batch, s);
            else launch_recurrent<float, kMlstm>(a, batch, s);
        } else {
            if (kind == kSsd) launch_recurrent<pa_bf16, kSsd>(a, batch, s);
            else launch_recurrent<pa_bf16, kMlstm>(a, batch, s);
        }
        PA_CHECK_LAUNCH("pa_gated_linear");
        return PA_OK;
    }
    a.segments = gl_plan(batch, num_heads, dim, vdim, max_q_len);
    while (a.segments > 1 && (!workspace || gl_workspace_bytes(batch, num_heads, dim, vdim, a.segments) > workspace_bytes))
        --a.segments;
    a.seg_rows = la_segment_rows(max_q_len, a.segments);
    a.ws = (float *)workspace;
    PA_REQUIRE(a.segments == 1 || pa_aligned16(workspace), "the workspace must be 16-byte aligned");
    return kind == kSsd ? launch_chunks_kind<kSsd>(a, batch, s) : launch_chunks_kind<kMlstm>(a, batch, s);
}
