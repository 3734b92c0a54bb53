// The gated delta rule: per head S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q, with S in 32-bit floats, kept
// per sequence in a pool of state slots.  q and k are made unit vectors here (q also times its scale), g and beta come from
// gate logits: g = exp(-rate softplus(raw + bias)), beta = sigmoid(raw).
//
// Two kernels, as for the other recurrences.  The recurrent one (a decode step, and 32-bit prompts) reads the state once,
// walks its rows token by token in registers and writes the state once.
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
    return 0;
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
    if (dtype == PA_F32) launch_delta_recurrent<float>(a, batch, s);
    else launch_delta_recurrent<pa_bf16>(a, batch, s);
    PA_CHECK_LAUNCH("pa_delta");
    return PA_OK;
}
