// The gated delta rule: per head S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q, with S in 32-bit floats, kept
// per sequence in a pool of state slots.  q and k are made unit vectors here (q also times its scale), g and beta come from
// gate logits: g = exp(-rate softplus(raw + bias)), beta = sigmoid(raw).
//
// Two kernels, as for the other recurrences.  The recurrent one (a decode step, and 32-bit prompts) reads the state once,
// walks its rows token by token in registers and writes the state once.
//
// Portions of 16-bit rows go in chunks of 64 on the matrix cores, in two passes.  With F the running sum of log decays in a
// chunk, all u of a chunk satisfy one triangular system: with A_ts = beta_t (k_t . k_s) e^(F_t - F_s) below the diagonal,
//     U = T (V - e^F K S),   T = (I + A)^-1 diag(beta),
//     O = e^F Q S + C U,     C_ts = (q_t . k_s) e^(F_t - F_s) for s <= t,
//     S <- e^(F_last) S + (e^(F_last - F) K)^T U.
// T and C do not depend on S: the first pass makes them for all chunks at once (T by inverting 16 x 16 blocks on the
// diagonal row by row and joining them with 32-bit matrix products).  The second pass walks a portion's chunks with S in
// accumulator registers; a wave owns value columns, which do not depend on each other.  Unit norms are factors of rows,
// so q and k enter the products as they are stored; T, C, S, U and V - e^F K S are split into two bf16 terms each.
#include "linear_tiles.h"

namespace {

constexpr float kUnitEps = 1e-6f;

struct DeltaArgs {
    const void *q, *k, *v;  // row strides ldq, ldk, ldv; head h: q, k at h / per_group * dim, v at h * vdim
    int64_t ldq, ldk, ldv;
    const void *ga, *gb;    // [row][head] at stride ldg: raw decay and beta logits
    int64_t ldg;
    const float *bias, *rate;  // [heads]
    float q_scale;
    int64_t n_rows;
    float *state;  // [state_rows][heads][dp][vp]
    int64_t state_rows;
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots;
    void *out;  // [rows][heads * vdim]
    char *ws;   // per chunk and head: DeltaChunk
    int heads, per_group, dim, vdim, dp, vp, chunks;  // chunks: most chunks of a portion
};

struct DeltaPortion {
    int n, pos0;
    int64_t row0, slot;
};
__device__ __forceinline__ bool delta_portion(const DeltaArgs &a, int b, DeltaPortion &p) {
    p.n = a.q_lens ? a.q_lens[b] : 1;
    p.row0 = a.q_starts ? a.q_starts[b] : b;
    p.pos0 = a.ctx_lens[b] - p.n;
    p.slot = a.state_slots[b];
    if (p.slot >= a.state_rows) p.slot = -1;
    return p.n > 0 && p.pos0 >= 0 && p.row0 >= 0 && p.row0 + p.n <= a.n_rows;
}

__device__ __forceinline__ float delta_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// Log decay to base 2
__device__ __forceinline__ float delta_log_decay(const DeltaArgs &a, int h, float raw) {
    return -a.rate[h] * delta_softplus(raw + a.bias[h]) * 1.4426950408889634f;
}
__device__ __forceinline__ float delta_sigmoid(float x) { return 1.f / (1.f + expf(-x)); }

// ------------------------------------------------------------------ token by token
constexpr int kDeltaCols = 64;  // value columns per workgroup: 16 lanes x float4, 16 groups of lanes over the rows of S

// R: rows of S per thread (16 R >= dim)
template <typename T, int R> __global__ __launch_bounds__(256, 4) void delta_recurrent_kernel(const DeltaArgs a) {
    __shared__ float qs[16 * R], ks[16 * R], vs[kDeltaCols];
    __shared__ float4 red[16][kDeltaCols / 4];
    __shared__ float redn[2][4];
    const int h = blockIdx.y, b = blockIdx.z, v0 = blockIdx.x * kDeltaCols;
    DeltaPortion p;
    if (!delta_portion(a, b, p)) return;
    const int tid = threadIdx.x, c4 = tid % 16, col = c4 * 4, grp = tid / 16;
    const bool live = v0 + col < a.vp;  // (vp is a multiple of 16)
    float *sp = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * (int64_t)a.dp * a.vp + v0 + col : nullptr;
    float4 s[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        s[r] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (sp && p.pos0 > 0 && live && d < a.dp) s[r] = *reinterpret_cast<const float4 *>(sp + (int64_t)d * a.vp);
    }
    const int g = h / a.per_group;
    const T *q = reinterpret_cast<const T *>(a.q) + g * a.dim, *k = reinterpret_cast<const T *>(a.k) + g * a.dim;
    const T *v = reinterpret_cast<const T *>(a.v) + h * a.vdim + v0;
    for (int t = 0; t < p.n; ++t) {
        const int64_t row = p.row0 + t;
        float qd = 0.f, kd = 0.f;
        if (tid < 16 * R) {  // (16 R <= 256)
            if (tid < a.dim) {
                qd = pa_scalar<T>::load(q + row * a.ldq + tid);
                kd = pa_scalar<T>::load(k + row * a.ldk + tid);
            }
            qs[tid] = qd;
            ks[tid] = kd;
        }
        if (tid < kDeltaCols) vs[tid] = v0 + tid < a.vdim ? pa_scalar<T>::load(v + row * a.ldv + tid) : 0.f;
        const float q2 = pa_group_sum<64>(qd * qd), k2 = pa_group_sum<64>(kd * kd);
        if (tid % 64 == 0) {
            redn[0][tid / 64] = q2;
            redn[1][tid / 64] = k2;
        }
        const float keep = exp2f(delta_log_decay(a, h, pa_scalar<T>::load(reinterpret_cast<const T *>(a.ga) + row * a.ldg + h)));
        const float beta = delta_sigmoid(pa_scalar<T>::load(reinterpret_cast<const T *>(a.gb) + row * a.ldg + h));
        __syncthreads();
        const float qn = a.q_scale / sqrtf(redn[0][0] + redn[0][1] + redn[0][2] + redn[0][3] + kUnitEps);
        const float kn = 1.f / sqrtf(redn[1][0] + redn[1][1] + redn[1][2] + redn[1][3] + kUnitEps);
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float f = ks[grp + 16 * r] * kn;
            s[r].x *= keep; s[r].y *= keep; s[r].z *= keep; s[r].w *= keep;
            x.x = fmaf(f, s[r].x, x.x); x.y = fmaf(f, s[r].y, x.y);
            x.z = fmaf(f, s[r].z, x.z); x.w = fmaf(f, s[r].w, x.w);
        }
        red[grp][c4] = x;
        __syncthreads();
        const float4 vv = *reinterpret_cast<const float4 *>(vs + col);
        float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const float4 y = red[i][c4];
            u.x += y.x; u.y += y.y; u.z += y.z; u.w += y.w;
        }
        u = make_float4(beta * (vv.x - u.x), beta * (vv.y - u.y), beta * (vv.z - u.z), beta * (vv.w - u.w));
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float f = ks[grp + 16 * r] * kn, e = qs[grp + 16 * r] * qn;
            s[r].x = fmaf(f, u.x, s[r].x); s[r].y = fmaf(f, u.y, s[r].y);
            s[r].z = fmaf(f, u.z, s[r].z); s[r].w = fmaf(f, u.w, s[r].w);
            o.x = fmaf(e, s[r].x, o.x); o.y = fmaf(e, s[r].y, o.y);
            o.z = fmaf(e, s[r].z, o.z); o.w = fmaf(e, s[r].w, o.w);
        }
        __syncthreads();  // red has been read
        red[grp][c4] = o;
        __syncthreads();
        if (tid < kDeltaCols && v0 + tid < a.vdim) {
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) sum += reinterpret_cast<const float *>(red[i])[tid];
            pa_scalar<T>::store(reinterpret_cast<T *>(a.out) + row * ((int64_t)a.heads * a.vdim) + h * a.vdim + v0 + tid, sum);
        }
        // (the next token's writes to qs, ks, vs and redn follow every thread's reads of them, before the barrier above; its
        // writes to red come after its own first barrier, which the threads that sum here reach afterwards)
    }
    if (!sp) return;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = grp + 16 * r;
        if (live && d < a.dp) *reinterpret_cast<float4 *>(sp + (int64_t)d * a.vp) = s[r];
    }
}

// ------------------------------------------------------------------ chunks: T and C
constexpr int kDcPitch = 72;  // bf16 per row of T and C in LDS
// Operands that meet a result as their partner have the inner order 4 g + 0 .. 3, 16 + 4 g + 0 .. 3 within 32: stored in that
// order, a lane's eight elements are one 16-byte chunk.  Position of element c:
__host__ __device__ constexpr int delta_paired(int c) { return (c & ~31) | (c & 12) << 1 | (c & 16) >> 2 | (c & 3); }
struct DeltaChunk {           // what the first pass leaves per chunk and head (columns of T and C paired)
    uint16_t t_hi[64][64], t_lo[64][64], c_hi[64][64], c_lo[64][64];
    float k_in[64];   // e^F times k's unit factor (on K S)
    float q_in[64];   // e^F times q's unit factor and scale (on Q S)
    float k_out[64];  // e^(F_last - F) times k's unit factor (on U in the new state)
    float keep;       // e^(F_last)
    float pad[63];
};

__device__ __forceinline__ f4 delta_mfma32(float x, float y, f4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, c, 0, 0, 0); }

// Inclusive sum over the wave
__device__ __forceinline__ float delta_scan(float x, int lane) {
#pragma unroll
    for (int d = 1; d < 64; d *= 2) {
        const float y = __shfl_up(x, d, 64);
        if (lane >= d) x += y;
    }
    return x;
}

// Workgroup: one chunk of one head.  Wave w: rows 16 w .. of the products.
template <int KD> __global__ __launch_bounds__(256, KD == 256 ? 2 : 4) void delta_prepare_kernel(const DeltaArgs a) {
    constexpr int kLd = KD + 8, kMat = 68, kRowBytes = 2 * 64 * kLd * 2, kMatBytes = 2 * 64 * kMat * 4;
    __shared__ __align__(16) char room[kRowBytes > kMatBytes ? kRowBytes : kMatBytes];
    __bf16 *q_s = reinterpret_cast<__bf16 *>(room), *k_s = q_s + 64 * kLd;
    // in their place once the products are made: A below the diagonal, (I + A)^-1
    float(*mat)[kMat] = reinterpret_cast<float(*)[kMat]>(room), (*inv)[kMat] = mat + 64;
    __shared__ float part[4][16][17];
    __shared__ float f_s[64], beta_s[64], kn_s[64], qn_s[64];
    const int h = blockIdx.x, chunk = blockIdx.y, b = blockIdx.z;
    DeltaPortion p;
    if (!delta_portion(a, b, p)) return;
    const int r0 = chunk * 64, nv = p.n - r0 < 64 ? p.n - r0 : 64;
    if (nv <= 0) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const int grp = h / a.per_group;
    const uint16_t *uq = reinterpret_cast<const uint16_t *>(a.q) + (p.row0 + r0) * a.ldq + grp * a.dim;
    const uint16_t *uk = reinterpret_cast<const uint16_t *>(a.k) + (p.row0 + r0) * a.ldk + grp * a.dim;
    {
        const __amdgpu_buffer_rsrc_t tq = la_tile(uq, a.ldq, nv, a.dim), tk = la_tile(uk, a.ldk, nv, a.dim);
        constexpr int kBlocks = 16 * (KD / 4), kPass = kBlocks / 256;
        static_assert(kBlocks % 256 == 0, "whole passes");
#pragma unroll
        for (int i = 0; i < kPass; ++i) {
            const int blk = tid + 256 * i, r = blk / (KD / 4) * 4, c = blk % (KD / 4) * 4;
            const LaBlock x = la_load_block(tq, la_block_off(a.ldq, r, c, a.dim), (uint32_t)a.ldq * 2u);
            const LaBlock y = la_load_block(tk, la_block_off(a.ldk, r, c, a.dim), (uint32_t)a.ldk * 2u);
            la_put_block<false>(x, r, c, q_s, kLd, nullptr);
            la_put_block<false>(y, r, c, k_s, kLd, nullptr);
        }
    }
    if (wave == 0) {
        float decay = 0.f, beta = 0.f;
        if (lane < nv) {
            const int64_t row = p.row0 + r0 + lane;
            decay = delta_log_decay(a, h, pa_scalar<pa_bf16>::load(reinterpret_cast<const pa_bf16 *>(a.ga) + row * a.ldg + h));
            beta = delta_sigmoid(pa_scalar<pa_bf16>::load(reinterpret_cast<const pa_bf16 *>(a.gb) + row * a.ldg + h));
        }
        f_s[lane] = delta_scan(decay, lane);
        beta_s[lane] = beta;
    }
    __syncthreads();
    {   // unit factors: four lanes per row
        const int r = tid / 4;
        float q2 = 0.f, k2 = 0.f;
#pragma unroll 4
        for (int d = tid % 4 * 8; d < KD; d += 32) {
            const bf8 x = la_read8(q_s + r * kLd + d), y = la_read8(k_s + r * kLd + d);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                q2 = fmaf((float)x[j], (float)x[j], q2);
                k2 = fmaf((float)y[j], (float)y[j], k2);
            }
        }
        q2 = pa_group_sum<4>(q2);
        k2 = pa_group_sum<4>(k2);
        if (tid % 4 == 0) {
            qn_s[r] = a.q_scale / sqrtf(q2 + kUnitEps);
            kn_s[r] = 1.f / sqrtf(k2 + kUnitEps);
        }
    }
    __syncthreads();
    DeltaChunk *out = reinterpret_cast<DeltaChunk *>(a.ws) + ((int64_t)b * a.chunks + chunk) * a.heads + h;
    if (tid < 64) {
        const float f = f_s[tid], last = f_s[63];
        out->k_in[tid] = exp2f(f) * kn_s[tid];
        out->q_in[tid] = exp2f(f) * qn_s[tid];
        out->k_out[tid] = exp2f(last - f) * kn_s[tid];
        if (tid == 0) out->keep = exp2f(last);
    }
    // rows t = 16 wave + l16 (as columns of the results), keys s = 16 st + 4 g + i
    f4 kk[4], qk[4];
#pragma unroll
    for (int st = 0; st < 4; ++st) kk[st] = qk[st] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int d = 0; d < KD / 32; ++d) {
        const bf8 bk = la_read8(k_s + (16 * wave + l16) * kLd + 32 * d + 8 * g), bq = la_read8(q_s + (16 * wave + l16) * kLd + 32 * d + 8 * g);
#pragma unroll
        for (int st = 0; st < 4; ++st) {
            if (st > wave) continue;
            const bf8 x = la_read8(k_s + (16 * st + l16) * kLd + 32 * d + 8 * g);
            kk[st] = la_mfma(x, bk, kk[st]);
            qk[st] = la_mfma(x, bq, qk[st]);
        }
    }
    __syncthreads();
    const int t = 16 * wave + l16;
    const float ft = f_s[t], bt = beta_s[t] * kn_s[t], qt = qn_s[t];
#pragma unroll
    for (int st = 0; st < 4; ++st) {
        float c[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int s = 16 * st + 4 * g + i;
            const float w = s <= t ? __builtin_amdgcn_exp2f(ft - f_s[s]) * kn_s[s] : 0.f;
            mat[t][s] = s < t ? kk[st][i] * w * bt : 0.f;
            c[i] = qk[st][i] * w * qt;
        }
        uint2 hi, lo;
        la_split2(c[0], c[1], hi.x, lo.x);
        la_split2(c[2], c[3], hi.y, lo.y);
        *reinterpret_cast<uint2 *>(&out->c_hi[t][delta_paired(16 * st + 4 * g)]) = hi;
        *reinterpret_cast<uint2 *>(&out->c_lo[t][delta_paired(16 * st + 4 * g)]) = lo;
    }
    // (the wave's own 16 rows of mat: its accesses are in order, the compiler must keep them so)
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    // diagonal block: column l16 of the inverse, row after row
    const int d0 = 16 * wave;
    if (lane < 16) {
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float y = i == l16 ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; ++j) y = fmaf(-mat[d0 + i][d0 + j], x[j], y);
            x[i] = y;
            inv[d0 + i][d0 + l16] = y;
        }
    }
    __syncthreads();
    // block (i, j), i - j = level: -inv_ii (sum over j <= k < i of mat_ik inv_kj)
    for (int level = 1; level < 4; ++level) {
        const int j = wave, i = wave + level;
        if (i < 4) {
            f4 x = f4{0.f, 0.f, 0.f, 0.f};
            for (int k = j; k < i; ++k)
#pragma unroll
                for (int q = 0; q < 4; ++q) x = delta_mfma32(mat[16 * i + l16][16 * k + 4 * q + g], inv[16 * k + 4 * q + g][16 * j + l16], x);
#pragma unroll
            for (int e = 0; e < 4; ++e) part[wave][4 * g + e][l16] = x[e];
            __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
            __builtin_amdgcn_wave_barrier();
            f4 y = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < 4; ++q) y = delta_mfma32(inv[16 * i + l16][16 * i + 4 * q + g], part[wave][4 * q + g][l16], y);
#pragma unroll
            for (int e = 0; e < 4; ++e) inv[16 * i + 4 * g + e][16 * j + l16] = -y[e];
        }
        __syncthreads();
    }
    for (int i = tid; i < 64 * 16; i += 256) {
        const int r = i / 16, c = i % 16 * 4;
        float x[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = c / 16 <= r / 16 ? inv[r][c + e] * beta_s[c + e] : 0.f;
        uint2 hi, lo;
        la_split2(x[0], x[1], hi.x, lo.x);
        la_split2(x[2], x[3], hi.y, lo.y);
        *reinterpret_cast<uint2 *>(&out->t_hi[r][delta_paired(c)]) = hi;
        *reinterpret_cast<uint2 *>(&out->t_lo[r][delta_paired(c)]) = lo;
    }
}

// ------------------------------------------------------------------ chunks: the walk
// Tiles of Q and K: paired columns, chunk c of row r at position c ^ delta_hash(r).  Operand reads (16 rows, one chunk) and
// transposing reads (four rows, four chunks) both spread over the banks.
template <int KD> __device__ __forceinline__ int delta_hash(int r) { return (KD == 64 ? (r & 2) << 1 : (r & 3) << 2) | (r >> 2 & 3); }
template <int KD> __device__ __forceinline__ void delta_put(const LaBlock &b, int r, int c, __bf16 *tile) {
    const int e = delta_paired(c);
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<uint2 *>(tile + (r + i) * KD + (((e >> 3) ^ delta_hash<KD>(r + i)) << 3) + (e & 4)) = b.r[i];
}

template <int KD, int COLS> constexpr size_t delta_walk_lds() {
    return (size_t)(2 * 64 * KD + 64 * (COLS + 8) + 4 * 64 * kDcPitch) * 2 + 3 * 64 * 4 + 64;
}

// Two bf16 terms of eight values of a result tile pair, as an operand whose inner index runs 4 g + 0 .. 3, then 16 more
__device__ __forceinline__ LaSplit delta_split(const f4 &x, const f4 &y) {
    LaSplit s;
    la_split2(x[0], x[1], s.hi[0], s.lo[0]);
    la_split2(x[2], x[3], s.hi[1], s.lo[1]);
    la_split2(y[0], y[1], s.hi[2], s.lo[2]);
    la_split2(y[2], y[3], s.hi[3], s.lo[3]);
    return s;
}

// KD: dim padded to 64, 128 or 256.  A workgroup of NW waves owns 16 NW value columns of a head and all chunks of a portion.
template <int KD, int NW> __global__ __launch_bounds__(64 * NW, 1) void delta_walk_kernel(const DeltaArgs a) {
    constexpr int kCols = 16 * NW, kThr = 64 * NW, kLv = kCols + 8;
    constexpr int kBlocks = 16 * (KD / 4), kKB = (kBlocks + kThr - 1) / kThr;  // 4 x 4 blocks of K, of V; 16-byte pieces of T and C
    constexpr int kVB = 16 * (kCols / 4) / kThr, kMB = 4 * 64 * 8 / kThr;
    static_assert(16 * (kCols / 4) % kThr == 0 && (kBlocks % kThr == 0 || kKB == 1), "whole passes");
    const bool k_live = kBlocks >= kThr || (int)threadIdx.x < kBlocks;
    extern __shared__ __align__(16) char lds[];
    __bf16 *q_s = reinterpret_cast<__bf16 *>(lds), *k_s = q_s + 64 * KD, *v_s = k_s + 64 * KD;
    __bf16 *m_s = v_s + 64 * kLv;  // T's two terms, C's two terms
    float *rows = reinterpret_cast<float *>(m_s + 4 * 64 * kDcPitch);  // k_in, q_in, k_out
    const __bf16 *t_hi = m_s, *t_lo = m_s + 64 * kDcPitch, *c_hi = m_s + 2 * 64 * kDcPitch, *c_lo = m_s + 3 * 64 * kDcPitch;
    const int h = blockIdx.x, v0 = blockIdx.y * kCols, b = blockIdx.z;
    DeltaPortion p;
    if (!delta_portion(a, b, p)) return;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), vw = wave * 16, l16 = tid & 15, g = (tid & 63) >> 4;
    // S: tile dt holds d = 16 dt + 4 g + i, v = v0 + vw + l16
    f4 s[KD / 16];
    const int64_t state_elems = (int64_t)a.dp * a.vp;
    float *pool = p.slot >= 0 ? a.state + (p.slot * a.heads + h) * state_elems : nullptr;
    const int v = v0 + vw + l16;
    const uint32_t soff = v < a.vp ? (uint32_t)(4 * g * a.vp + v) * 4u : kLaOutside;
    {
        const float *from = p.pos0 > 0 ? pool : nullptr;
        const __amdgpu_buffer_rsrc_t src = __builtin_amdgcn_make_buffer_rsrc((void *)(from ? from : a.state), 0, from ? (int)state_elems * 4 : 0, 0x00020000);
#pragma unroll
        for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                s[dt][i] = __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(src, soff + (16 * dt + i) * a.vp * 4, 0, 0));
    }
    const int grp = h / a.per_group;
    const uint16_t *uq = reinterpret_cast<const uint16_t *>(a.q) + p.row0 * a.ldq + grp * a.dim;
    const uint16_t *uk = reinterpret_cast<const uint16_t *>(a.k) + p.row0 * a.ldk + grp * a.dim;
    const uint16_t *uv = reinterpret_cast<const uint16_t *>(a.v) + p.row0 * a.ldv + h * a.vdim + v0;
    const int vcols = a.vdim - v0 < kCols ? a.vdim - v0 : kCols;
    const DeltaChunk *mats = reinterpret_cast<const DeltaChunk *>(a.ws) + (int64_t)b * a.chunks * a.heads + h;
    LaBlock qb[kKB], kb[kKB], vb[kVB];
    la_u4 mb[kMB];
    float keep_next = 0.f, row_g0 = 0.f, row_g1 = 0.f, row_g2 = 0.f;
    auto fetch = [&](int r0) {
        const int nr = p.n - r0 < 64 ? p.n - r0 : 64;
        const __amdgpu_buffer_rsrc_t tq = la_tile(uq + r0 * a.ldq, a.ldq, nr, a.dim), tk = la_tile(uk + r0 * a.ldk, a.ldk, nr, a.dim);
        const __amdgpu_buffer_rsrc_t tv = la_tile(uv + r0 * a.ldv, a.ldv, nr, vcols);
#pragma unroll
        for (int i = 0; i < kKB; ++i) {
            const int blk = tid + kThr * i, r = blk / (KD / 4) * 4, c = blk % (KD / 4) * 4;
            qb[i] = la_load_block(tq, k_live ? la_block_off(a.ldq, r, c, a.dim) : kLaOutside, (uint32_t)a.ldq * 2u);
            kb[i] = la_load_block(tk, k_live ? la_block_off(a.ldk, r, c, a.dim) : kLaOutside, (uint32_t)a.ldk * 2u);
        }
#pragma unroll
        for (int i = 0; i < kVB; ++i) {
            const int blk = tid + kThr * i, r = blk / (kCols / 4) * 4, c = blk % (kCols / 4) * 4;
            vb[i] = la_load_block(tv, la_block_off(a.ldv, r, c, vcols), (uint32_t)a.ldv * 2u);
        }
        const DeltaChunk *m = mats + (int64_t)(r0 / 64) * a.heads;
#pragma unroll
        for (int i = 0; i < kMB; ++i) mb[i] = reinterpret_cast<const la_u4 *>(m)[tid + kThr * i];
        row_g0 = m->k_in[tid & 63];
        row_g1 = m->q_in[tid & 63];
        row_g2 = m->k_out[tid & 63];
        keep_next = m->keep;
    };
    fetch(0);
    for (int r0 = 0; r0 < p.n; r0 += 64) {
        const int nv = p.n - r0 < 64 ? p.n - r0 : 64;
#pragma unroll
        for (int i = 0; i < kKB; ++i) {
            const int blk = tid + kThr * i, r = blk / (KD / 4) * 4, c = blk % (KD / 4) * 4;
            if (!k_live) continue;
            delta_put<KD>(qb[i], r, c, q_s);
            delta_put<KD>(kb[i], r, c, k_s);
        }
#pragma unroll
        for (int i = 0; i < kVB; ++i) {
            const int blk = tid + kThr * i, r = blk / (kCols / 4) * 4, c = blk % (kCols / 4) * 4;
            la_put_block<false>(vb[i], r, c, v_s, kLv, nullptr);
        }
#pragma unroll
        for (int i = 0; i < kMB; ++i) {
            const int at = tid + kThr * i;  // 16-byte piece: row at / 8 over the four matrices
            *reinterpret_cast<la_u4 *>(m_s + at / 8 * kDcPitch + at % 8 * 8) = mb[i];
        }
        if (tid < 64) {
            rows[tid] = row_g0;
            rows[64 + tid] = row_g1;
            rows[128 + tid] = row_g2;
        }
        const float keep = keep_next;
        if (r0 + 64 < p.n) fetch(r0 + 64);
        __syncthreads();
        // K S (rows t = 16 tt + 4 g + i, columns v) and, transposed, Q S (v = 4 g + i of the wave's columns, t = 16 tt + l16)
        f4 u[4], o[4];
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) u[tt] = o[tt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int dd = 0; dd < KD / 32; ++dd) {
            const LaSplit sp = delta_split(s[2 * dd], s[2 * dd + 1]);
            const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
            for (int tt = 0; tt < 4; ++tt) {
                const int at = (16 * tt + l16) * KD + ((4 * dd + g) ^ delta_hash<KD>(l16)) * 8;
                const bf8 xk = la_read8(k_s + at), xq = la_read8(q_s + at);
                u[tt] = la_mfma(xk, hi, u[tt]);
                u[tt] = la_mfma(xk, lo, u[tt]);
                o[tt] = la_mfma(hi, xq, o[tt]);
                o[tt] = la_mfma(lo, xq, o[tt]);
            }
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
            const f4 ki = *reinterpret_cast<const f4 *>(rows + 16 * tt + 4 * g);
            const la_bf4 vv = la_read_tr(v_s + (16 * tt + 4 * g + l16 / 4) * kLv + vw + l16 % 4 * 4);
            const float qi = rows[64 + 16 * tt + l16];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                u[tt][i] = (float)vv[i] - ki[i] * u[tt][i];
                o[tt][i] *= qi;
            }
        }
        // U = T R
        f4 w[4];
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) w[tt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const LaSplit sp = delta_split(u[2 * kk], u[2 * kk + 1]);
            const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
            for (int tt = 2 * kk; tt < 4; ++tt) {
                const int at = (16 * tt + l16) * kDcPitch + 32 * kk + 8 * g;
                const bf8 th = la_read8(t_hi + at), tl = la_read8(t_lo + at);
                w[tt] = la_mfma(th, hi, w[tt]);
                w[tt] = la_mfma(th, lo, w[tt]);
                w[tt] = la_mfma(tl, hi, w[tt]);
            }
        }
        // O += C U (transposed), S <- keep S + K^T (k_out U)
#pragma unroll
        for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i) s[dt][i] *= keep;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            {
                const LaSplit sp = delta_split(w[2 * kk], w[2 * kk + 1]);
                const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
                for (int tt = 2 * kk; tt < 4; ++tt) {
                    const int at = (16 * tt + l16) * kDcPitch + 32 * kk + 8 * g;
                    const bf8 ch = la_read8(c_hi + at), cl = la_read8(c_lo + at);
                    o[tt] = la_mfma(hi, ch, o[tt]);
                    o[tt] = la_mfma(lo, ch, o[tt]);
                    o[tt] = la_mfma(hi, cl, o[tt]);
                }
            }
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                const f4 ko = *reinterpret_cast<const f4 *>(rows + 128 + 32 * kk + 16 * half + 4 * g);
#pragma unroll
                for (int i = 0; i < 4; ++i) w[2 * kk + half][i] *= ko[i];
            }
            const LaSplit sp = delta_split(w[2 * kk], w[2 * kk + 1]);
            const bf8 hi = sp.high(), lo = sp.low();
#pragma unroll
            for (int dt = 0; dt < KD / 16; ++dt) {
                const int row = 4 * g + l16 / 4;
                const __bf16 *at = k_s + (32 * kk + row) * KD + ((dt / 2 * 4 + l16 % 4) ^ delta_hash<KD>(row)) * 8 + dt % 2 * 4;
                const bf8 xk = la_join(la_read_tr(at), la_read_tr(at + 16 * KD));
                s[dt] = la_mfma(xk, hi, s[dt]);
                s[dt] = la_mfma(xk, lo, s[dt]);
            }
        }
        const int ldo = a.heads * a.vdim, c = vw + 4 * g;
        const uint16_t *first = reinterpret_cast<const uint16_t *>(a.out) + (p.row0 + r0) * (int64_t)ldo + h * a.vdim + v0;
        const __amdgpu_buffer_rsrc_t dst = la_tile(first, ldo, nv, vcols);
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
            const la_u2 x = {row_pack_bf16(o[tt][0], o[tt][1]), row_pack_bf16(o[tt][2], o[tt][3])};
            __builtin_amdgcn_raw_buffer_store_b64(x, dst, c < vcols ? (uint32_t)((16 * tt + l16) * ldo + c) * 2u : kLaOutside, 0, 0);
        }
        __syncthreads();  // the next chunk's tiles may be written now
    }
    if (!pool) return;
    const __amdgpu_buffer_rsrc_t dst = __builtin_amdgcn_make_buffer_rsrc((void *)pool, 0, (int)state_elems * 4, 0x00020000);
#pragma unroll
    for (int dt = 0; dt < KD / 16; ++dt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float f = s[dt][i];
            __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(uint32_t, f), dst, soff + (16 * dt + i) * a.vp * 4, 0, 0);
        }
}

template <int KD, int NW> int launch_walk(const DeltaArgs &a, int batch, hipStream_t s) {
    constexpr size_t lds = delta_walk_lds<KD, 16 * NW>();
    static_assert(lds <= 160 * 1024, "LDS of one compute unit");
    if (int rc = la_big_lds(delta_walk_kernel<KD, NW>, lds, "pa_delta")) return rc;
    delta_walk_kernel<KD, NW><<<dim3((unsigned)a.heads, (unsigned)((a.vdim + 16 * NW - 1) / (16 * NW)), (unsigned)batch), dim3(64 * NW), lds, s>>>(a);
    PA_CHECK_LAUNCH("pa_delta (chunks)");
    return PA_OK;
}

template <int KD> int launch_delta_chunks(const DeltaArgs &a, int batch, hipStream_t s) {
    delta_prepare_kernel<KD><<<dim3((unsigned)a.heads, (unsigned)a.chunks, (unsigned)batch), dim3(256), 0, s>>>(a);
    PA_CHECK_LAUNCH("pa_delta (triangular systems)");
    // the widest slices of the value columns that leave no compute unit without one
    const int64_t heads = (int64_t)batch * a.heads;
    // (at dim 256 four waves' registers hold the state and the next chunk)
    if constexpr (KD == 256) {
        return launch_walk<KD, 4>(a, batch, s);
    } else {
        if (a.vdim > 64 && heads * ((a.vdim + 127) / 128) >= la_cus()) return launch_walk<KD, 8>(a, batch, s);
        if (a.vdim > 32 && heads * ((a.vdim + 63) / 64) >= la_cus()) return launch_walk<KD, 4>(a, batch, s);
        return launch_walk<KD, 2>(a, batch, s);
    }
}

size_t delta_ws_bytes(int batch, int heads, int max_q_len) { return (size_t)batch * heads * ((max_q_len + 63) / 64) * sizeof(DeltaChunk); }

template <typename T> void launch_delta_recurrent(const DeltaArgs &a, int batch, hipStream_t s) {
    const dim3 grid((unsigned)((a.vdim + kDeltaCols - 1) / kDeltaCols), (unsigned)a.heads, (unsigned)batch), block(256);
    if (a.dim <= 64) delta_recurrent_kernel<T, 4><<<grid, block, 0, s>>>(a);
    else if (a.dim <= 128) delta_recurrent_kernel<T, 8><<<grid, block, 0, s>>>(a);
    else delta_recurrent_kernel<T, 16><<<grid, block, 0, s>>>(a);
}

}  // namespace

extern "C" size_t pa_delta_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len) {
    pa_clear_error();
    if (batch < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || max_q_len < 0) {
        pa_fail(PA_ERR_INVALID_ARG, "pa_delta_workspace_bytes: sizes out of range");
        return 0;
    }
    return dim > 256 ? 0 : delta_ws_bytes(batch, num_heads, max_q_len);
}

extern "C" int pa_delta(const void *q, int64_t q_stride, const void *k, int64_t k_stride, const void *v, int64_t v_stride,
                        int heads_per_group, const void *decay_logits, const void *beta_logits, int64_t gate_stride,
                        const float *decay_bias, const float *decay_rate, float q_scale, int64_t n_rows, float *state,
                        int64_t state_rows, const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                        const int32_t *state_slots, int batch, int max_q_len, void *out, int num_heads, int dim, int vdim,
                        int dtype, void *workspace, size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && state_rows >= 0 && max_q_len >= 0, "pa_delta: a count is negative");
    PA_REQUIRE(num_heads > 0 && dim > 0 && vdim > 0, "pa_delta: heads / dim / vdim must be positive");
    PA_REQUIRE(heads_per_group > 0 && num_heads % heads_per_group == 0, "heads_per_group=%d does not divide num_heads=%d",
               heads_per_group, num_heads);
    PA_REQUIRE(num_heads <= 65535 && batch <= 65535, "pa_delta: heads=%d / batch=%d above 65535", num_heads, batch);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_delta: dtype=%d is not F32 or BF16", dtype);
    if (dim > 256) return pa_fail(PA_ERR_UNSUPPORTED, "pa_delta: dim=%d above 256", dim);
    const int groups = num_heads / heads_per_group;
    PA_REQUIRE(q_stride >= (int64_t)groups * dim && k_stride >= (int64_t)groups * dim && v_stride >= (int64_t)num_heads * vdim &&
                   gate_stride >= num_heads, "pa_delta: a stride is shorter than its row");
    PA_REQUIRE((int64_t)num_heads * (dim + vdim) <= 0x7fffffff, "pa_delta: rows are too long");
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "pa_delta: q_lens and q_starts come together");
    if (n_rows == 0 || batch == 0 || (q_lens && max_q_len == 0)) return PA_OK;
    PA_REQUIRE(q && k && v && decay_logits && beta_logits && decay_bias && decay_rate && state && ctx_lens && state_slots && out,
               "pa_delta: NULL argument");
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    PA_REQUIRE(pa_aligned16(state), "pa_delta: the state must be 16-byte aligned");
    DeltaArgs a{};
    a.q = q; a.k = k; a.v = v; a.ldq = q_stride; a.ldk = k_stride; a.ldv = v_stride; a.per_group = heads_per_group;
    a.ga = decay_logits; a.gb = beta_logits; a.ldg = gate_stride; a.bias = decay_bias; a.rate = decay_rate; a.q_scale = q_scale;
    a.n_rows = n_rows; a.state = state; a.state_rows = state_rows; a.ctx_lens = ctx_lens; a.q_lens = q_lens;
    a.q_starts = q_starts; a.state_slots = state_slots; a.out = out; a.heads = num_heads; a.dim = dim; a.vdim = vdim;
    a.dp = la_pad16(dim); a.vp = la_pad16(vdim);
    hipStream_t s = (hipStream_t)stream;
    // (single rows, 32-bit rows, rows that are not whole 8-byte vectors, rows too far apart for 32-bit offsets go one by one)
    const uintptr_t at = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)out;
    const int64_t most = 1 << 22;
    if (q_lens && dtype == PA_BF16 && workspace && workspace_bytes >= delta_ws_bytes(batch, num_heads, max_q_len) && pa_aligned16(workspace) &&
        dim % 4 == 0 && vdim % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && v_stride % 4 == 0 && (at & 7u) == 0 && q_stride <= most &&
        k_stride <= most && v_stride <= most && (int64_t)num_heads * vdim <= most && (max_q_len + 63) / 64 <= 65535) {
        a.ws = (char *)workspace;
        a.chunks = (max_q_len + 63) / 64;
        return dim <= 64 ? launch_delta_chunks<64>(a, batch, s) : dim <= 128 ? launch_delta_chunks<128>(a, batch, s) : launch_delta_chunks<256>(a, batch, s);
    }
    if (dtype == PA_F32) launch_delta_recurrent<float>(a, batch, s);
    else launch_delta_recurrent<pa_bf16>(a, batch, s);
    PA_CHECK_LAUNCH("pa_delta");
    return PA_OK;
}
