// Short causal convolution over time, one filter per channel, with bias, silu and carried rows: the step between a
// recurrent layer's projection and its recurrence.  HBM-bound: every projected value is read once (a tile's first rows
// twice), everything between is in 32-bit registers.
//
// Work item: (tile of up to kTile rows of one sequence, eight channels).  As in qkv_append.hip the tile that starts a
// portion is the only one that reads the carried rows, and after reading them into registers it writes the new ones.
#include "row_common.h"

namespace {

constexpr int kTile = PA_QKV_TILE_ROWS;

struct ConvArgs {
    const void *u;  // [rows][ldu]
    int64_t ldu;
    const float *w, *bias;  // [taps][channels], [channels] or NULL
    void *state;            // [state_rows][taps - 1][channels] of T
    int64_t state_rows;
    const int32_t *ctx_lens, *q_lens, *q_starts, *state_slots, *tiles;
    void *out;  // [rows][channels]
    int64_t n_rows;
    int channels, taps, batch, act;
};

template <typename T, bool VEC> __device__ __forceinline__ void conv_load(const T *p, int n, float *f) {
    if constexpr (VEC) {
        row_load<T, 8>(p, f);
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] = i < n ? pa_scalar<T>::load(p + i) : 0.f;
    }
}
template <typename T, bool VEC> __device__ __forceinline__ void conv_store(T *p, int n, const float *f) {
    if constexpr (VEC) {
        row_store<T, 8>(p, f);
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < n) pa_scalar<T>::store(p + i, f[i]);
    }
}

// HT: rows of history held in registers (taps - 1 <= HT; the missing leading taps have weight zero).
template <typename T, int HT, bool VEC> __global__ __launch_bounds__(256) void conv_kernel(const ConvArgs a) {
    const int c0 = (blockIdx.y * 256 + threadIdx.x) * 8;
    if (c0 >= a.channels) return;
    const int left = a.channels - c0 < 8 ? a.channels - c0 : 8;
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
    const T *u = reinterpret_cast<const T *>(a.u) + c0;
    const int keep = a.taps - 1;  // carried rows

    float w[HT + 1][8], hist[HT][8], bias[8];
#pragma unroll
    for (int j = 0; j <= HT; ++j) {
        const int tap = j - (HT - keep);
        row_zero<8>(w[j]);
        if (tap >= 0) conv_load<float, VEC>(a.w + (int64_t)tap * a.channels + c0, left, w[j]);
    }
    row_zero<8>(bias);
    if (a.bias) conv_load<float, VEC>(a.bias + c0, left, bias);
    int64_t sslot = a.state && a.state_slots ? a.state_slots[b] : -1;
    if (sslot >= a.state_rows) sslot = -1;
    T *state = sslot >= 0 ? reinterpret_cast<T *>(a.state) + sslot * keep * a.channels + c0 : nullptr;
#pragma unroll
    for (int j = 0; j < HT; ++j) {
        const int idx = i0 - HT + j;    // row of the portion
        const int srow = idx + keep;    // row of the carried state when it lies before the portion
        row_zero<8>(hist[j]);
        if (j < HT - keep) continue;    // weight zero
        if (idx >= 0) conv_load<T, VEC>(u + (row0 + idx) * a.ldu, left, hist[j]);
        else if (state && pos0 > 0 && srow >= 0) conv_load<T, VEC>(state + (int64_t)srow * a.channels, left, hist[j]);
    }
    if (i0 == 0 && state) {  // the last taps - 1 projected rows so far
#pragma unroll
        for (int j = 0; j < HT; ++j) {
            const int srow = j - (HT - keep);
            if (srow < 0) continue;
            const int idx = n - HT + j;
            float f[8];
            row_zero<8>(f);
            if (idx >= 0) {
                conv_load<T, VEC>(u + (row0 + idx) * a.ldu, left, f);
            } else {
#pragma unroll
                for (int m = 0; m < HT; ++m)
                    if (m == HT + idx)
#pragma unroll
                        for (int e = 0; e < 8; ++e) f[e] = hist[m][e];
            }
            conv_store<T, VEC>(state + (int64_t)srow * a.channels, left, f);
        }
    }
    T *out = reinterpret_cast<T *>(a.out) + c0;
    for (int i = i0; i < i1; ++i) {
        float cur[8], y[8];
        conv_load<T, VEC>(u + (row0 + i) * a.ldu, left, cur);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float acc = bias[e];
#pragma unroll
            for (int j = 0; j < HT; ++j) acc = fmaf(w[j][e], hist[j][e], acc);
            acc = fmaf(w[HT][e], cur[e], acc);
            y[e] = a.act == PA_ACT_SILU ? row_silu<T>(acc) : acc;
        }
        conv_store<T, VEC>(out + (row0 + i) * a.channels, left, y);
#pragma unroll
        for (int j = 0; j + 1 < HT; ++j)
#pragma unroll
            for (int e = 0; e < 8; ++e) hist[j][e] = hist[j + 1][e];
#pragma unroll
        for (int e = 0; e < 8; ++e) hist[HT - 1][e] = cur[e];
    }
}

template <typename T> void launch_conv(const ConvArgs &a, int n_tiles, bool vec, hipStream_t s) {
    const dim3 grid((unsigned)n_tiles, (unsigned)((a.channels + 2047) / 2048)), block(256);
    if (!vec) conv_kernel<T, 7, false><<<grid, block, 0, s>>>(a);
    else if (a.taps <= 4) conv_kernel<T, 3, true><<<grid, block, 0, s>>>(a);
    else conv_kernel<T, 7, true><<<grid, block, 0, s>>>(a);
}

}  // namespace

extern "C" int pa_short_conv(const void *u, int64_t u_stride, int64_t n_rows, const float *weight, const float *bias, int taps,
                             int act, void *conv_state, int64_t state_rows, const int32_t *ctx_lens, const int32_t *q_lens,
                             const int32_t *q_starts, const int32_t *state_slots, const int32_t *tiles, int n_tiles,
                             int batch, void *out, int channels, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && n_tiles >= 0 && state_rows >= 0, "pa_short_conv: a count is negative");
    PA_REQUIRE(channels > 0 && taps >= 1, "pa_short_conv: channels=%d / taps=%d must be positive", channels, taps);
    PA_REQUIRE(act == PA_ACT_NONE || act == PA_ACT_SILU, "act=%d is unknown", act);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_short_conv: dtype=%d is not F32 or BF16", dtype);
    if (taps > 8) return pa_fail(PA_ERR_UNSUPPORTED, "pa_short_conv: taps=%d above 8", taps);
    PA_REQUIRE(u_stride >= channels, "u_stride=%lld is shorter than the channels", (long long)u_stride);
    PA_REQUIRE(tiles || n_tiles == batch, "without tiles every sequence brings one row");
    PA_REQUIRE(tiles || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    if (n_rows == 0 || n_tiles == 0) return PA_OK;
    PA_REQUIRE(u && weight && ctx_lens && out, "NULL argument");
    PA_REQUIRE(!tiles || (q_lens && q_starts), "tiles without q_lens / q_starts");
    PA_REQUIRE(taps == 1 || (conv_state && state_slots), "a convolution needs its carried state");
    ConvArgs a{u, u_stride, weight, bias, taps > 1 ? conv_state : nullptr, state_rows, ctx_lens, q_lens, q_starts, state_slots,
               tiles, out, n_rows, channels, taps, batch, act};
    const bool vec = channels % 8 == 0 && u_stride % 8 == 0 && pa_aligned16(u) && pa_aligned16(weight) && pa_aligned16(bias) &&
                     pa_aligned16(conv_state) && pa_aligned16(out);
    if (dtype == PA_F32) launch_conv<float>(a, n_tiles, vec, (hipStream_t)stream);
    else launch_conv<pa_bf16>(a, n_tiles, vec, (hipStream_t)stream);
    PA_CHECK_LAUNCH("pa_short_conv");
    return PA_OK;
}
