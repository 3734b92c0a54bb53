// Row kernels between the matrix products of a decoder block: the 32-bit residual sum fused with the norm that
// reads it, gated activations, and the gates behind attention and recurrent layers.  HBM-bound; a row lives in
// registers, every tensor is read once and written once.
#include "row_common.h"

namespace {

// ------------------------------------------------------------------ residual sum + norm
struct ResidualArgs {
    float *x;               // [rows][width], the residual stream (read and, with y or ids, written)
    const void *y;          // branch output [rows][width] of T, or NULL
    const float *y_weight;  // RMS norm applied to y before the sum, or NULL
    const int64_t *ids;     // x starts as table[ids[row]], or NULL
    const void *table;
    int64_t table_rows;
    const int64_t *row_index;  // output row r reads residual row row_index[r] (x is not written), or NULL
    int64_t x_rows;
    const float *w, *b;  // norm weight and bias
    void *out;           // [rows][width] of T, or NULL
    int64_t rows;
    int width, norm;
    float y_eps, eps;
};

template <typename T, int TPR, int V, int NV>
__global__ __launch_bounds__(256) void residual_norm_kernel(const ResidualArgs a) {
    __shared__ float red[8];
    const int64_t row = (int64_t)blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
    if (row >= a.rows) return;  // (uniform over the TPR threads that share a row)
    const int lane = threadIdx.x % TPR;
    int64_t xrow = row;
    bool have_x = true;
    if (a.row_index) {
        xrow = a.row_index[row];
        have_x = xrow >= 0 && xrow < a.x_rows;
    }
    float x[NV][V];
    if (a.ids) {
        const int64_t id = a.ids[row];
        const bool ok = id >= 0 && id < a.table_rows;
        const T *src = reinterpret_cast<const T *>(a.table) + (ok ? id : 0) * a.width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            row_zero<V>(x[i]);
            if (ok && c < a.width) row_load<T, V>(src + c, x[i]);
        }
    } else {
        const float *src = a.x + (have_x ? xrow : 0) * a.width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            row_zero<V>(x[i]);
            if (have_x && c < a.width) row_load<float, V>(src + c, x[i]);
        }
    }
    if (a.y) {
        const T *src = reinterpret_cast<const T *>(a.y) + row * a.width;
        float y[NV][V];
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            row_zero<V>(y[i]);
            if (c < a.width) row_load<T, V>(src + c, y[i]);
        }
        if (a.y_weight) {
            float ss = 0.f;
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int j = 0; j < V; ++j) ss = fmaf(y[i][j], y[i][j], ss);
            const float inv = 1.f / sqrtf(row_sum<TPR>(ss, red) / (float)a.width + a.y_eps);
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * TPR + lane) * V;
                float w[V];
                row_zero<V>(w);
                if (c < a.width) row_load<float, V>(a.y_weight + c, w);
#pragma unroll
                for (int j = 0; j < V; ++j) x[i][j] += y[i][j] * inv * w[j];
            }
        } else {
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int j = 0; j < V; ++j) x[i][j] += y[i][j];
        }
    }
    if (a.x && !a.row_index && (a.y || a.ids)) {
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            if (c < a.width) row_store<float, V>(a.x + row * a.width + c, x[i]);
        }
    }
    if (!a.out) return;
    float mean = 0.f, inv = 1.f;
    if (a.norm == PA_NORM_LAYER) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int j = 0; j < V; ++j) s += x[i][j];
        mean = row_sum<TPR>(s, red) / (float)a.width;
    }
    if (a.norm != PA_NORM_NONE) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
#pragma unroll
            for (int j = 0; j < V; ++j) {
                const float d = c + j < a.width ? x[i][j] - mean : 0.f;
                ss = fmaf(d, d, ss);
            }
        }
        inv = 1.f / sqrtf(row_sum<TPR>(ss, red) / (float)a.width + a.eps);
    }
    T *dst = reinterpret_cast<T *>(a.out) + row * a.width;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        if (c >= a.width) continue;
        float w[V], b[V], o[V];
        row_fill<V>(w, 1.f);
        row_zero<V>(b);
        if (a.w) row_load<float, V>(a.w + c, w);
        if (a.b) row_load<float, V>(a.b + c, b);
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] = (x[i][j] - mean) * inv * w[j] + b[j];
        row_store<T, V>(dst + c, o);
    }
}

// ------------------------------------------------------------------ RMS norm + sigmoid gate
struct RmsGateArgs {
    const void *o;  // [rows][width] of T
    const void *g;  // gate logits, row stride ldg
    int64_t ldg;
    const float *w;
    void *out;  // [rows][width]
    int64_t rows;
    int width;
    float eps;
};

template <typename T, int TPR, int V, int NV>
__global__ __launch_bounds__(256) void rms_gate_kernel(const RmsGateArgs a) {
    __shared__ float red[8];
    const int64_t row = (int64_t)blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
    if (row >= a.rows) return;
    const int lane = threadIdx.x % TPR;
    const T *src = reinterpret_cast<const T *>(a.o) + row * a.width;
    const T *gate = reinterpret_cast<const T *>(a.g) + row * a.ldg;
    float x[NV][V], g[NV][V];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        row_zero<V>(x[i]);
        row_zero<V>(g[i]);
        if (c < a.width) {
            row_load<T, V>(src + c, x[i]);
            row_load<T, V>(gate + c, g[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < V; ++j) ss = fmaf(x[i][j], x[i][j], ss);
    const float inv = 1.f / sqrtf(row_sum<TPR>(ss, red) / (float)a.width + a.eps);
    T *dst = reinterpret_cast<T *>(a.out) + row * a.width;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        if (c >= a.width) continue;
        float w[V], o[V];
        row_load<float, V>(a.w + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] = x[i][j] * inv * w[j] * row_sigmoid<T>(g[i][j]);
        row_store<T, V>(dst + c, o);
    }
}

// ------------------------------------------------------------------ elementwise
struct GluArgs {
    const void *gate, *up;  // [rows] of strides ldg, ldu
    int64_t ldg, ldu;
    const int64_t *ids;  // the factor of row r is row ids[r] of `up`, or NULL: row r
    int64_t up_rows;
    void *out;  // [rows][width]
    int64_t rows;
    int width, act;
};

// out = act(gate) * up; with ids the second factor is a row of a table (the per-layer token input)
template <typename T, int V> __global__ __launch_bounds__(256) void glu_kernel(const GluArgs a) {
    const int per_row = (a.width + V - 1) / V;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t row = i / per_row;
    if (row >= a.rows) return;
    const int c = (int)(i - row * per_row) * V;
    int64_t urow = row;
    bool ok = true;
    if (a.ids) {
        urow = a.ids[row];
        ok = urow >= 0 && urow < a.up_rows;
        if (!ok) urow = 0;
    }
    float g[V], u[V], o[V];
    row_load<T, V>(reinterpret_cast<const T *>(a.gate) + row * a.ldg + c, g);
    row_load<T, V>(reinterpret_cast<const T *>(a.up) + urow * a.ldu + c, u);
#pragma unroll
    for (int j = 0; j < V; ++j)
        o[j] = (a.act == PA_ACT_SILU ? g[j] * row_sigmoid<T>(g[j]) : row_gelu_tanh<T>(g[j])) * (ok ? u[j] : 0.f);
    row_store<T, V>(reinterpret_cast<T *>(a.out) + row * a.width + c, o);
}

struct HeadGateArgs {
    const void *o;  // [rows][heads][d]
    const void *g;  // one logit per head, row stride ldg
    int64_t ldg;
    void *out;  // [rows][heads][vdim]
    int64_t rows;
    int heads, d, vdim;
};

// out = o * sigmoid(gate of the head), the first vdim of every head's d values, packed
template <typename T, int V> __global__ __launch_bounds__(256) void head_gate_kernel(const HeadGateArgs a) {
    const int per_head = a.vdim / V, per_row = a.heads * per_head;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t row = i / per_row;
    if (row >= a.rows) return;
    const int r = (int)(i - row * per_row), h = r / per_head, c = (r - h * per_head) * V;
    float o[V];
    row_load<T, V>(reinterpret_cast<const T *>(a.o) + (row * a.heads + h) * a.d + c, o);
    if (a.g) {
        const float s = row_sigmoid<T>(pa_scalar<T>::load(reinterpret_cast<const T *>(a.g) + row * a.ldg + h));
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] *= s;
    }
    row_store<T, V>(reinterpret_cast<T *>(a.out) + (row * a.heads + h) * a.vdim + c, o);
}

// Threads per row and registers per thread by row width: one wave up to 1024 columns, a workgroup above.
#define ROW_DISPATCH(KERNEL, T, vec4, width, rows, args, s)                                                \
    do {                                                                                                   \
        const unsigned grid64_ = (unsigned)(((rows) + 3) / 4), grid256_ = (unsigned)(rows);                \
        if (!(vec4)) KERNEL<T, 256, 1, 64><<<dim3(grid256_), dim3(256), 0, s>>>(args);                     \
        else if ((width) <= 256) KERNEL<T, 64, 4, 1><<<dim3(grid64_), dim3(256), 0, s>>>(args);            \
        else if ((width) <= 512) KERNEL<T, 64, 4, 2><<<dim3(grid64_), dim3(256), 0, s>>>(args);            \
        else if ((width) <= 1024) KERNEL<T, 256, 4, 1><<<dim3(grid256_), dim3(256), 0, s>>>(args);         \
        else if ((width) <= 2048) KERNEL<T, 256, 4, 2><<<dim3(grid256_), dim3(256), 0, s>>>(args);         \
        else if ((width) <= 4096) KERNEL<T, 256, 4, 4><<<dim3(grid256_), dim3(256), 0, s>>>(args);         \
        else if ((width) <= 8192) KERNEL<T, 256, 4, 8><<<dim3(grid256_), dim3(256), 0, s>>>(args);         \
        else KERNEL<T, 256, 4, 16><<<dim3(grid256_), dim3(256), 0, s>>>(args);                             \
    } while (0)

constexpr int kMaxWidth = 16384;

int check_rows(const char *what, int64_t rows, int width, int dtype) {
    PA_REQUIRE(rows >= 0 && width > 0, "%s: rows=%lld / width=%d out of range", what, (long long)rows, width);
    PA_REQUIRE(rows <= 0x7fffffff, "%s: rows=%lld is too large for one launch", what, (long long)rows);
    if (width > kMaxWidth) return pa_fail(PA_ERR_UNSUPPORTED, "%s: width=%d above %d", what, width, kMaxWidth);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "%s: dtype=%d is not F32 or BF16", what, dtype);
    return PA_OK;
}

}  // namespace

extern "C" int pa_residual_norm(float *x, const void *y, const float *y_weight, float y_eps, const int64_t *ids,
                                const void *table, int64_t table_rows, const int64_t *row_index, int64_t x_rows,
                                const float *norm_weight, const float *norm_bias, float eps, int norm, void *out,
                                int64_t rows, int width, int dtype, void *stream) {
    pa_clear_error();
    if (int rc = check_rows("pa_residual_norm", rows, width, dtype)) return rc;
    PA_REQUIRE(norm == PA_NORM_NONE || norm == PA_NORM_LAYER || norm == PA_NORM_RMS, "norm=%d is unknown", norm);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x || ids, "neither a residual nor an embedding to start from");
    PA_REQUIRE(!ids || table, "ids without a table");
    PA_REQUIRE(!row_index || (x && !y && !ids), "row_index only reads the residual");
    PA_REQUIRE(!y_weight || y, "y_weight without y");
    PA_REQUIRE(out || (x && (y || ids)), "nothing to write");
    PA_REQUIRE(norm != PA_NORM_NONE || (!norm_weight && !norm_bias), "norm weights without a norm");
    ResidualArgs a{x, y, y_weight, ids, table, table_rows, row_index, x_rows, norm_weight, norm_bias, out, rows, width,
                   norm, y_eps, eps};
    const bool vec4 = width % 4 == 0 && pa_aligned16(x) && pa_aligned16(y) && pa_aligned16(table) && pa_aligned16(out) &&
                      pa_aligned16(y_weight) && pa_aligned16(norm_weight) && pa_aligned16(norm_bias);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) ROW_DISPATCH(residual_norm_kernel, float, vec4, width, rows, a, s);
    else ROW_DISPATCH(residual_norm_kernel, pa_bf16, vec4, width, rows, a, s);
    PA_CHECK_LAUNCH("pa_residual_norm");
    return PA_OK;
}

extern "C" int pa_rms_gate(const void *o, const void *gate, int64_t gate_stride, const float *weight, float eps, void *out,
                           int64_t rows, int width, int dtype, void *stream) {
    pa_clear_error();
    if (int rc = check_rows("pa_rms_gate", rows, width, dtype)) return rc;
    if (rows == 0) return PA_OK;
    PA_REQUIRE(o && gate && weight && out, "NULL argument");
    PA_REQUIRE(gate_stride >= width, "gate_stride=%lld is shorter than a row", (long long)gate_stride);
    RmsGateArgs a{o, gate, gate_stride, weight, out, rows, width, eps};
    const uintptr_t gmask = dtype == PA_F32 ? 15u : 7u;  // four elements
    const bool vec4 = width % 4 == 0 && gate_stride % 4 == 0 && ((uintptr_t)gate & gmask) == 0 && pa_aligned16(o) &&
                      pa_aligned16(weight) && pa_aligned16(out);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) ROW_DISPATCH(rms_gate_kernel, float, vec4, width, rows, a, s);
    else ROW_DISPATCH(rms_gate_kernel, pa_bf16, vec4, width, rows, a, s);
    PA_CHECK_LAUNCH("pa_rms_gate");
    return PA_OK;
}

extern "C" int pa_glu(const void *gate, int64_t gate_stride, const void *up, int64_t up_stride, const int64_t *ids,
                      int64_t up_rows, void *out, int64_t rows, int width, int act, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && width > 0, "pa_glu: rows=%lld / width=%d out of range", (long long)rows, width);
    PA_REQUIRE(act == PA_ACT_SILU || act == PA_ACT_GELU_TANH, "act=%d is unknown", act);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_glu: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(gate && up && out, "NULL argument");
    PA_REQUIRE(gate_stride >= width && up_stride >= width, "a stride is shorter than a row");
    GluArgs a{gate, up, gate_stride, up_stride, ids, up_rows, out, rows, width, act};
    const int n = dtype == PA_F32 ? 4 : 8;
    const bool vec = width % n == 0 && gate_stride % n == 0 && up_stride % n == 0 && pa_aligned16(gate) && pa_aligned16(up) &&
                     pa_aligned16(out);
    const int64_t items = rows * (vec ? width / n : width), grid = (items + 255) / 256;
    PA_REQUIRE(grid <= 0x7fffffff, "pa_glu: rows=%lld is too large for one launch", (long long)rows);
    const dim3 g((unsigned)grid), blk(256);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) {
        if (vec) glu_kernel<float, 4><<<g, blk, 0, s>>>(a);
        else glu_kernel<float, 1><<<g, blk, 0, s>>>(a);
    } else {
        if (vec) glu_kernel<pa_bf16, 8><<<g, blk, 0, s>>>(a);
        else glu_kernel<pa_bf16, 1><<<g, blk, 0, s>>>(a);
    }
    PA_CHECK_LAUNCH("pa_glu");
    return PA_OK;
}

extern "C" int pa_head_gate(const void *o, const void *gate, int64_t gate_stride, void *out, int64_t rows, int heads, int d,
                            int vdim, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && heads > 0 && d > 0 && vdim > 0 && vdim <= d, "pa_head_gate: sizes out of range");
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_head_gate: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(o && out, "NULL argument");
    PA_REQUIRE(!gate || gate_stride >= heads, "gate_stride=%lld is shorter than a row", (long long)gate_stride);
    HeadGateArgs a{o, gate, gate_stride, out, rows, heads, d, vdim};
    const int n = dtype == PA_F32 ? 4 : 8;
    const bool vec = d % n == 0 && vdim % n == 0 && pa_aligned16(o) && pa_aligned16(out);
    const int64_t items = rows * heads * (vec ? vdim / n : vdim), grid = (items + 255) / 256;
    PA_REQUIRE(grid <= 0x7fffffff, "pa_head_gate: rows=%lld is too large for one launch", (long long)rows);
    const dim3 g((unsigned)grid), blk(256);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) {
        if (vec) head_gate_kernel<float, 4><<<g, blk, 0, s>>>(a);
        else head_gate_kernel<float, 1><<<g, blk, 0, s>>>(a);
    } else {
        if (vec) head_gate_kernel<pa_bf16, 8><<<g, blk, 0, s>>>(a);
        else head_gate_kernel<pa_bf16, 1><<<g, blk, 0, s>>>(a);
    }
    PA_CHECK_LAUNCH("pa_head_gate");
    return PA_OK;
}
