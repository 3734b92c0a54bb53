// From the joint q/k/v projection to attention's operands in one pass: a short causal convolution over time with its
// carried state, RMS norms of q and k, interleaved rotary positions on the leading dimensions, value mixing, and the
// append of k and v to the paged pool.  HBM-bound: every projected value is read once, everything between is in
// 32-bit registers.
//
// Work item: (tile of up to kTile rows of one sequence, head).  LPH lanes hold one head, eight channels each, and walk
// the tile's rows with the last projected rows in registers.  The tile that starts a sequence's portion is the only
// one that reads the carried rows, and it also writes the new ones (after reading them into registers), so one
// launch needs no second buffer: the portion's later tiles find their history in the projections themselves.
#include "row_common.h"

namespace {

constexpr int kTile = PA_QKV_TILE_ROWS;
constexpr int kThreadsQkv = 256;

struct QkvArgs {
    const void *u;  // [rows][ldu]: hq * dim of q, hkv * dim of k, hkv * vdim of v, anything
    int64_t ldu;
    const float *bias;    // [channels], or NULL (only without a convolution)
    const float *conv_w;  // [taps][channels], or NULL (taps == 1)
    void *conv_state;     // [state_rows][taps - 1][channels] of T
    int64_t state_rows;
    const float2 *rope;  // [rope_rows][rot / 2]: (cos, sin)
    int64_t rope_rows;
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots, *tiles;
    const int64_t *slots;
    int64_t total_slots, n_rows;
    void *q_out;  // [rows][hq][d]
    void *k_cache, *v_cache;  // [total_slots][hkv][d]
    void *v_first;            // [rows][hkv * vdim]
    const float *lambda;
    const float *q_norm, *k_norm;  // [dim]: weights of RMS norms ahead of the rotation, or NULL
    int v_mode, batch, hq, hkv, dim, vdim, d, taps, rot, unit_norm;
    float eps, q_scale;
};

// Eight channels from `p`, of which `n` exist (vector loads only where VEC says the layout allows them).
template <typename T, bool VEC> __device__ __forceinline__ void load8(const T *p, int n, float *f) {
    if constexpr (VEC) {
        if (n > 0) row_load<T, 8>(p, f);
        else row_zero<8>(f);
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] = i < n ? pa_scalar<T>::load(p + i) : 0.f;
    }
}
template <typename T, bool VEC> __device__ __forceinline__ void store8(T *p, int n, const float *f) {
    if constexpr (VEC) {
        if (n > 0) row_store<T, 8>(p, f);
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) pa_scalar<T>::store(p + i, f[i]);
    }
}

// HT: rows of history held in registers (taps - 1 <= HT; the missing leading taps have weight zero).
template <typename T, int LPH, int HT, bool VEC>
__global__ __launch_bounds__(kThreadsQkv) void qkv_append_kernel(const QkvArgs a) {
    const int unit = blockIdx.y * (kThreadsQkv / LPH) + threadIdx.x / LPH;
    const int units = a.hq + 2 * a.hkv;
    if (unit >= units) return;
    const int lane = threadIdx.x % LPH, c0 = lane * 8;
    int b, i0 = 0, n = 1;
    int64_t row0;
    if (a.tiles) {
        b = a.tiles[2 * blockIdx.x];
        i0 = a.tiles[2 * blockIdx.x + 1];
        if (b < 0 || b >= a.batch) return;
        n = a.q_lens[b];
        row0 = a.q_starts[b];
    } else {
        b = blockIdx.x;
        row0 = b;
    }
    const int pos0 = a.ctx_lens[b] - n;  // position of the portion's first row
    if (pos0 < 0 || i0 < 0 || i0 >= n || row0 < 0 || row0 + n > a.n_rows) return;
    const int i1 = i0 + kTile < n ? i0 + kTile : n;

    const bool is_q = unit < a.hq, is_v = unit >= a.hq + a.hkv;
    const int head = is_q ? unit : (is_v ? unit - a.hq - a.hkv : unit - a.hq);
    const int width = is_v ? a.vdim : a.dim;
    const int chan = (is_v ? (a.hq + a.hkv) * a.dim + head * a.vdim : unit * a.dim) + c0;
    const int left = width - c0 < 0 ? 0 : (width - c0 > 8 ? 8 : width - c0);  // channels of this lane that exist
    const int channels = (a.hq + a.hkv) * a.dim + a.hkv * a.vdim;
    const T *u = reinterpret_cast<const T *>(a.u) + chan;

    float w[HT + 1][8], hist[HT][8];
#pragma unroll
    for (int j = 0; j <= HT; ++j) {
        const int tap = j - (HT + 1 - a.taps);
        row_fill<8>(w[j], j == HT ? 1.f : 0.f);
        if (a.conv_w && tap >= 0) load8<float, VEC>(a.conv_w + (int64_t)tap * channels + chan, left, w[j]);
        if (a.conv_w && tap < 0) row_zero<8>(w[j]);
    }
    int64_t sslot = -1;
    if (a.conv_state && a.state_slots) {
        sslot = a.state_slots[b];
        if (sslot >= a.state_rows) sslot = -1;
    }
    T *state = sslot >= 0 ? reinterpret_cast<T *>(a.conv_state) + sslot * (a.taps - 1) * channels + chan : nullptr;
#pragma unroll
    for (int j = 0; j < HT; ++j) {
        const int idx = i0 - HT + j;           // row of the portion
        const int srow = idx + a.taps - 1;     // row of the carried state when it lies before the portion
        row_zero<8>(hist[j]);
        if (j < HT - (a.taps - 1)) continue;   // weight zero
        if (idx >= 0) load8<T, VEC>(u + (row0 + idx) * a.ldu, left, hist[j]);
        else if (state && pos0 > 0 && srow >= 0) load8<T, VEC>(state + (int64_t)srow * channels, left, hist[j]);
    }
    if (i0 == 0 && state) {  // the last taps - 1 projected rows so far
#pragma unroll
        for (int j = 0; j < HT; ++j) {
            const int srow = j - (HT - (a.taps - 1));
            if (srow < 0) continue;
            const int idx = n - HT + j;
            float f[8];
            row_zero<8>(f);
            if (idx >= 0) {
                load8<T, VEC>(u + (row0 + idx) * a.ldu, left, f);
            } else {
#pragma unroll
                for (int m = 0; m < HT; ++m)
                    if (m == HT + idx)
#pragma unroll
                        for (int e = 0; e < 8; ++e) f[e] = hist[m][e];
            }
            store8<T, VEC>(state + (int64_t)srow * channels, left, f);
        }
    }

    const float lam = is_v && a.v_mode == PA_V_MIX ? *a.lambda : 0.f;
    const float *norm_w = is_v ? nullptr : is_q ? a.q_norm : a.k_norm;
    float nw[8];
    row_zero<8>(nw);
    if (norm_w) load8<float, VEC>(norm_w + c0, left, nw);
    float bias[8];
    row_zero<8>(bias);
    if (a.bias) load8<float, VEC>(a.bias + chan, left, bias);
    const int half = a.rot / 2;
    for (int i = i0; i < i1; ++i) {
        const int64_t row = row0 + i;
        float cur[8], y[8];
        load8<T, VEC>(u + row * a.ldu, left, cur);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float acc = 0.f;
#pragma unroll
            for (int j = 0; j < HT; ++j) acc = fmaf(w[j][e], hist[j][e], acc);
            y[e] = fmaf(w[HT][e], cur[e], acc + bias[e]);
        }
#pragma unroll
        for (int j = 0; j + 1 < HT; ++j)
#pragma unroll
            for (int e = 0; e < 8; ++e) hist[j][e] = hist[j + 1][e];
#pragma unroll
        for (int e = 0; e < 8; ++e) hist[HT - 1][e] = cur[e];

        if (is_v) {
            if (a.v_mode != PA_V_PLAIN) {
                T *vf = reinterpret_cast<T *>(a.v_first) + row * ((int64_t)a.hkv * a.vdim) + head * a.vdim + c0;
                if (a.v_mode == PA_V_FIRST) {
                    store8<T, VEC>(vf, left, y);
                } else {
                    float f[8];
                    load8<T, VEC>(vf, left, f);
#pragma unroll
                    for (int e = 0; e < 8; ++e) y[e] = (1.f - lam) * y[e] + lam * f[e];
                }
            }
        } else {
            if (norm_w) {
                float ss = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) ss = fmaf(y[e], y[e], ss);
                const float inv = 1.f / sqrtf(pa_group_sum<LPH>(ss) / (float)a.dim + a.eps);
#pragma unroll
                for (int e = 0; e < 8; ++e) y[e] *= inv * nw[e];
            }
            if (c0 < a.rot) {
                int64_t pos = pos0 + i;
                if (pos >= a.rope_rows) pos = a.rope_rows - 1;  // (the caller sizes the table; never read past it)
                const float2 *cs = a.rope + pos * half + c0 / 2;
#pragma unroll
                for (int p = 0; p < 4; ++p) {
                    if (c0 + 2 * p < a.rot) {
                        const float2 t = cs[p];
                        const float x0 = y[2 * p], x1 = y[2 * p + 1];
                        y[2 * p] = x0 * t.x - x1 * t.y;
                        y[2 * p + 1] = x1 * t.x + x0 * t.y;
                    }
                }
            }
            float f = is_q ? a.q_scale : 1.f;
            if (a.unit_norm) {
                float ss = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) ss = fmaf(y[e], y[e], ss);
                ss = pa_group_sum<LPH>(ss);
                f *= 1.f / sqrtf(ss / (float)a.dim + a.eps);
            }
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] *= f;
        }
        if (c0 >= a.d) continue;  // (lanes past the pool row; the channels between width and d are zeros)
        if (is_q) {
            row_store<T, 8>(reinterpret_cast<T *>(a.q_out) + (row * a.hq + head) * a.d + c0, y);
        } else {
            const int64_t slot = a.slots[row];
            if (slot < 0 || slot >= a.total_slots) continue;
            T *pool = reinterpret_cast<T *>(is_v ? a.v_cache : a.k_cache);
            row_store<T, 8>(pool + (slot * a.hkv + head) * a.d + c0, y);
        }
    }
}

template <typename T, int LPH> void launch_qkv(const QkvArgs &a, int n_tiles, bool vec, hipStream_t s) {
    const int per_wg = kThreadsQkv / LPH;
    const dim3 grid((unsigned)n_tiles, (unsigned)((a.hq + 2 * a.hkv + per_wg - 1) / per_wg)), block(kThreadsQkv);
    if (!vec) qkv_append_kernel<T, LPH, 7, false><<<grid, block, 0, s>>>(a);
    else if (a.taps <= 4) qkv_append_kernel<T, LPH, 3, true><<<grid, block, 0, s>>>(a);
    else qkv_append_kernel<T, LPH, 7, true><<<grid, block, 0, s>>>(a);
}

template <typename T> void launch_qkv_typed(const QkvArgs &a, int n_tiles, bool vec, hipStream_t s) {
    if (a.d <= 32) launch_qkv<T, 4>(a, n_tiles, vec, s);
    else if (a.d <= 64) launch_qkv<T, 8>(a, n_tiles, vec, s);
    else if (a.d <= 128) launch_qkv<T, 16>(a, n_tiles, vec, s);
    else launch_qkv<T, 32>(a, n_tiles, vec, s);
}

}  // namespace

extern "C" int pa_qkv_conv_append(const void *u, int64_t u_stride, int64_t n_rows, const float *bias, const float *conv_weight, int taps,
                                  void *conv_state, int64_t state_rows, const float *rope, int64_t rope_rows, int rot_dims,
                                  const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                                  const int32_t *state_slots, const int32_t *tiles, int n_tiles, int batch,
                                  const int64_t *slots, int64_t total_slots, void *q_out, void *k_cache, void *v_cache,
                                  void *v_first, const float *v_lambda, int v_mode, const float *q_norm,
                                  const float *k_norm, int num_q_heads, int num_kv_heads, int dim, int vdim, int pool_dim,
                                  int unit_norm, float eps, float q_scale, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && n_tiles >= 0 && total_slots >= 0 && state_rows >= 0 && rope_rows >= 0,
               "a count is negative");
    PA_REQUIRE(num_q_heads > 0 && num_kv_heads > 0 && num_q_heads % num_kv_heads == 0,
               "num_q_heads=%d must be a positive multiple of num_kv_heads=%d", num_q_heads, num_kv_heads);
    PA_REQUIRE(dim > 0 && vdim > 0 && pool_dim >= dim && pool_dim >= vdim && pool_dim % 8 == 0,
               "pool_dim=%d must be a multiple of 8 that holds dim=%d and vdim=%d", pool_dim, dim, vdim);
    PA_REQUIRE(rot_dims >= 0 && rot_dims <= dim && rot_dims % 2 == 0, "rot_dims=%d must be even and at most dim=%d", rot_dims, dim);
    PA_REQUIRE(taps >= 1 && (taps == 1 || conv_weight), "taps=%d without convolution weights", taps);
    PA_REQUIRE(!bias || taps == 1, "a bias ahead of a convolution");
    PA_REQUIRE(v_mode == PA_V_PLAIN || v_mode == PA_V_FIRST || v_mode == PA_V_MIX, "v_mode=%d is unknown", v_mode);
    if (dtype != PA_F32 && dtype != PA_BF16)
        return pa_fail(PA_ERR_UNSUPPORTED, "pa_qkv_conv_append: dtype=%d is not F32 or BF16", dtype);
    if (pool_dim > 256) return pa_fail(PA_ERR_UNSUPPORTED, "pa_qkv_conv_append: pool_dim=%d above 256", pool_dim);
    if (taps > 8) return pa_fail(PA_ERR_UNSUPPORTED, "pa_qkv_conv_append: taps=%d above 8", taps);
    const int64_t channels = (int64_t)(num_q_heads + num_kv_heads) * dim + (int64_t)num_kv_heads * vdim;
    PA_REQUIRE(u_stride >= channels && channels <= 0x7fffffff, "u_stride=%lld is shorter than q, k and v", (long long)u_stride);
    PA_REQUIRE(tiles || n_tiles == batch, "without tiles every sequence brings one row");
    PA_REQUIRE(tiles || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    if (n_rows == 0 || n_tiles == 0) return PA_OK;
    PA_REQUIRE(u && ctx_lens && slots && q_out && k_cache && v_cache, "NULL argument");
    PA_REQUIRE(!tiles || (q_lens && q_starts), "tiles without q_lens / q_starts");
    PA_REQUIRE(rot_dims == 0 || (rope && rope_rows > 0), "rot_dims=%d without a table", rot_dims);
    PA_REQUIRE(taps == 1 || (conv_state && state_slots), "a convolution needs its carried state");
    PA_REQUIRE(v_mode == PA_V_PLAIN || v_first, "v_mode without v_first");
    PA_REQUIRE(v_mode != PA_V_MIX || v_lambda, "value mixing without v_lambda");
    PA_REQUIRE((q_norm == nullptr) == (k_norm == nullptr), "q_norm and k_norm come together");
    PA_REQUIRE(pa_aligned16(q_out) && pa_aligned16(k_cache) && pa_aligned16(v_cache), "pointers must be 16-byte aligned");
    QkvArgs a{};
    a.u = u; a.ldu = u_stride; a.bias = bias; a.conv_w = conv_weight; a.conv_state = taps > 1 ? conv_state : nullptr;
    a.state_rows = state_rows; a.rope = (const float2 *)rope; a.rope_rows = rope_rows;
    a.ctx_lens = ctx_lens; a.q_lens = q_lens; a.q_starts = q_starts; a.state_slots = state_slots; a.tiles = tiles;
    a.slots = slots; a.total_slots = total_slots; a.n_rows = n_rows; a.q_out = q_out; a.k_cache = k_cache;
    a.v_cache = v_cache; a.v_first = v_first; a.lambda = v_lambda; a.v_mode = v_mode; a.batch = batch;
    a.hq = num_q_heads; a.hkv = num_kv_heads; a.dim = dim; a.vdim = vdim; a.d = pool_dim; a.taps = taps; a.rot = rot_dims;
    a.q_norm = q_norm; a.k_norm = k_norm; a.unit_norm = unit_norm; a.eps = eps; a.q_scale = q_scale;
    const bool vec = dim % 8 == 0 && vdim % 8 == 0 && u_stride % 8 == 0 && pa_aligned16(u) && pa_aligned16(bias) && pa_aligned16(conv_weight) &&
                     pa_aligned16(conv_state) && pa_aligned16(v_first) && pa_aligned16(q_norm) && pa_aligned16(k_norm);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) launch_qkv_typed<float>(a, n_tiles, vec, s);
    else launch_qkv_typed<pa_bf16>(a, n_tiles, vec, s);
    PA_CHECK_LAUNCH("pa_qkv_conv_append");
    return PA_OK;
}
