// Residual streams with learned mixing (hyper-connections) around the sublayers of a decoder block.  One pass over a row
// ends a sublayer and starts the next one: the streams are mixed with the branch's output, written back, summed under the
// next sublayer's weights and normed.  HBM-bound: every stream is read once and written once.
#include "row_common.h"

namespace {

constexpr int kMaxStreams = 16;

struct HyperArgs {
    float *x;            // [rows][streams][width]
    const void *y;       // branch output [rows][width] of T (with mix_w: [rows * mix][width]), or NULL
    const float *mix_w;  // [rows][mix_ld]: y = sum of mix_w[i] y[row * mix + i], i < mix, + mix_w[mix] y_extra + mix_w[mix + 1] y_self
    const void *y_extra, *y_self;  // [rows][width] of T, or NULL
    int mix, mix_ld;
    const float *between, *into;  // the branch that ends: [streams from][streams to], [streams]
    const int64_t *ids;           // the streams start as table[ids[row]], or NULL
    const void *table;
    int64_t table_rows;
    const float *weights;  // [streams]: what is summed for `out` and `sum`; NULL: ones
    const float *norm_w;
    void *out;    // [rows][width] of T: the normed sum, or NULL
    float *sum;   // [rows][width]: the sum as it is, or NULL
    int64_t rows;
    int streams, width;
    float eps;
};

// S: streams held (the loops over them are unrolled; those past `streams` are skipped).  TPR threads share a row.
template <typename T, int TPR, int V, int NV, int S>
__global__ __launch_bounds__(256) void hyper_kernel(const HyperArgs a) {
    __shared__ float red[8];
    __shared__ float between[kMaxStreams * kMaxStreams], into[kMaxStreams], weights[kMaxStreams];
    const int n = a.streams, tid = threadIdx.x;
    for (int i = tid; i < n * n; i += 256) between[i] = a.y ? a.between[i] : 0.f;
    if (tid < n) {
        into[tid] = a.y ? a.into[tid] : 0.f;
        weights[tid] = a.weights ? a.weights[tid] : 1.f;
    }
    __syncthreads();
    const int64_t row = (int64_t)blockIdx.x * (256 / TPR) + tid / TPR;
    if (row >= a.rows) return;  // (uniform over the TPR threads that share a row)
    const int lane = tid % TPR;
    int64_t id = -1;
    if (a.ids) {
        id = a.ids[row];
        if (id >= a.table_rows) id = -1;
    }
    const float *mw = a.mix_w ? a.mix_w + row * a.mix_ld : nullptr;
    float *xr = a.x + row * n * (int64_t)a.width;
    float u[NV][V], ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        row_zero<V>(u[i]);
        if (c >= a.width) continue;
        float x[S][V], y[V];
        if (a.ids) {
            float t[V];
            row_zero<V>(t);
            if (id >= 0) row_load<T, V>(reinterpret_cast<const T *>(a.table) + id * a.width + c, t);
#pragma unroll
            for (int s = 0; s < S; ++s)
#pragma unroll
                for (int j = 0; j < V; ++j) x[s][j] = t[j];
        } else {
#pragma unroll
            for (int s = 0; s < S; ++s) {
                row_zero<V>(x[s]);
                if (s < n) row_load<float, V>(xr + (int64_t)s * a.width + c, x[s]);
            }
        }
        if (a.y) {
            row_zero<V>(y);
            if (mw) {
                auto add = [&](const void *from, int64_t r, float f) {
                    if (f == 0.f) return;  // (an item that no product has written)
                    float t[V];
                    row_load<T, V>(reinterpret_cast<const T *>(from) + r * a.width + c, t);
#pragma unroll
                    for (int j = 0; j < V; ++j) y[j] = fmaf(f, t[j], y[j]);
                };
#pragma unroll 4
                for (int m = 0; m < a.mix; ++m) add(a.y, row * a.mix + m, mw[m]);
                if (a.y_extra) add(a.y_extra, row, mw[a.mix]);
                if (a.y_self) add(a.y_self, row, mw[a.mix + 1]);
            } else {
                row_load<T, V>(reinterpret_cast<const T *>(a.y) + row * a.width + c, y);
            }
        }
#pragma unroll
        for (int t = 0; t < S; ++t) {
            if (t >= n) continue;
            float z[V];
            if (a.y) {
#pragma unroll
                for (int j = 0; j < V; ++j) z[j] = into[t] * y[j];
#pragma unroll
                for (int s = 0; s < S; ++s) {
                    if (s >= n) continue;
                    const float f = between[s * n + t];
#pragma unroll
                    for (int j = 0; j < V; ++j) z[j] = fmaf(f, x[s][j], z[j]);
                }
            } else {
#pragma unroll
                for (int j = 0; j < V; ++j) z[j] = x[t][j];
            }
            if ((a.y && !a.sum) || a.ids) row_store<float, V>(xr + (int64_t)t * a.width + c, z);
            const float w = weights[t];
#pragma unroll
            for (int j = 0; j < V; ++j) u[i][j] = fmaf(w, z[j], u[i][j]);
        }
#pragma unroll
        for (int j = 0; j < V; ++j) ss = fmaf(u[i][j], u[i][j], ss);
        if (a.sum) row_store<float, V>(a.sum + row * a.width + c, u[i]);
    }
    if (!a.out) return;
    const float inv = 1.f / sqrtf(row_sum<TPR>(ss, red) / (float)a.width + a.eps);
    T *dst = reinterpret_cast<T *>(a.out) + row * a.width;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        if (c >= a.width) continue;
        float w[V];
        row_load<float, V>(a.norm_w + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) u[i][j] *= inv * w[j];
        row_store<T, V>(dst + c, u[i]);
    }
}

template <typename T, int S> void launch_hyper(const HyperArgs &a, bool vec4, hipStream_t s) {
    const dim3 b(256), per4((unsigned)((a.rows + 3) / 4)), per1((unsigned)a.rows);
    if (!vec4) hyper_kernel<T, 256, 1, 64, S><<<per1, b, 0, s>>>(a);
    else if (a.width <= 256) hyper_kernel<T, 64, 4, 1, S><<<per4, b, 0, s>>>(a);
    else if (a.width <= 512) hyper_kernel<T, 64, 4, 2, S><<<per4, b, 0, s>>>(a);
    else if (a.width <= 1024) hyper_kernel<T, 256, 4, 1, S><<<per1, b, 0, s>>>(a);
    else if (a.width <= 2048) hyper_kernel<T, 256, 4, 2, S><<<per1, b, 0, s>>>(a);
    else if (a.width <= 4096) hyper_kernel<T, 256, 4, 4, S><<<per1, b, 0, s>>>(a);
    else hyper_kernel<T, 256, 4, 16, S><<<per1, b, 0, s>>>(a);
}

template <typename T> void launch_hyper_typed(const HyperArgs &a, bool vec4, hipStream_t s) {
    if (a.streams <= 2) launch_hyper<T, 2>(a, vec4, s);
    else if (a.streams <= 4) launch_hyper<T, 4>(a, vec4, s);
    else if (a.streams <= 8) launch_hyper<T, 8>(a, vec4, s);
    else launch_hyper<T, kMaxStreams>(a, vec4, s);
}

}  // namespace

extern "C" int pa_hyper_norm(float *x, const void *y, const float *mix_weight, int mix, int mix_stride, const void *y_extra,
                             const void *y_self, const float *between, const float *into, const int64_t *ids, const void *table,
                             int64_t table_rows, const float *sum_weight, const float *norm_weight, float eps, void *out,
                             float *sum, int64_t rows, int streams, int width, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && width > 0 && streams > 0, "pa_hyper_norm: sizes out of range");
    PA_REQUIRE(rows <= 0x7fffffff, "pa_hyper_norm: rows=%lld is too large for one launch", (long long)rows);
    if (width > 16384 || streams > kMaxStreams)
        return pa_fail(PA_ERR_UNSUPPORTED, "pa_hyper_norm: width=%d above 16384 or streams=%d above %d", width, streams, kMaxStreams);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_hyper_norm: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x, "pa_hyper_norm: NULL streams");
    PA_REQUIRE(!ids || (table && !y), "pa_hyper_norm: ids without a table, or beside y");
    PA_REQUIRE(!y || (between && into), "pa_hyper_norm: y without its weights");
    PA_REQUIRE(!mix_weight || (y && mix > 0 && mix_stride >= mix + (y_self ? 2 : y_extra ? 1 : 0)), "pa_hyper_norm: mix_weight does not fit");
    PA_REQUIRE((!y_extra && !y_self) || mix_weight, "pa_hyper_norm: y_extra / y_self without mix_weight");
    PA_REQUIRE(!out || norm_weight, "pa_hyper_norm: out without norm_weight");
    PA_REQUIRE(out || sum || ids || y, "pa_hyper_norm: nothing to write");
    HyperArgs a{};
    a.x = x; a.y = y; a.mix_w = mix_weight; a.mix = mix; a.mix_ld = mix_stride; a.y_extra = y_extra; a.y_self = y_self;
    a.between = between; a.into = into; a.ids = ids; a.table = table; a.table_rows = table_rows; a.weights = sum_weight;
    a.norm_w = norm_weight; a.eps = eps; a.out = out; a.sum = sum; a.rows = rows; a.streams = streams; a.width = width;
    const bool vec4 = width % 4 == 0 && pa_aligned16(x) && pa_aligned16(y) && pa_aligned16(y_extra) && pa_aligned16(y_self) &&
                      pa_aligned16(table) && pa_aligned16(norm_weight) && pa_aligned16(out) && pa_aligned16(sum);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) launch_hyper_typed<float>(a, vec4, s);
    else launch_hyper_typed<pa_bf16>(a, vec4, s);
    PA_CHECK_LAUNCH("pa_hyper_norm");
    return PA_OK;
}
