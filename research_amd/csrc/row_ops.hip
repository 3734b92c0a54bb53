// Row kernels between the matrix products of a decoder block: the 32-bit residual sum fused with the norm that
// reads it, gated activations, and the gates behind attention and recurrent layers.  HBM-bound; a row lives in
// registers, every tensor is read once and written once.
#include "row_common.h"

namespace {

// ------------------------------------------------------------------ residual sum + norm
struct ResidualArgs {
    float *x;               // [rows][width], the residual stream (read and, with y or ids, written)
    const void *y;          // branch output [rows][width] of T (with mix_w: [rows * mix][width]), or NULL
    const float *mix_w;     // [rows][mix + 1]: y = sum of mix_w[i] y[row * mix + i], i < mix, + mix_w[mix] y_extra[row]
    const void *y_extra;    // [rows][width] of T, or NULL: without the last term
    int mix;
    const float *y_bias;    // added to y, or NULL
    const void *y2;         // a second branch, [rows][width] of T: y = y / rms(y) y_part + y2 / rms(y2) y2_part, or NULL
    const float *y_part, *y2_part;
    const float *y_weight;  // RMS norm applied to y before the sum, or NULL
    const int64_t *ids;     // x starts as table[ids[row]] (ids_add: gets it added), or NULL
    int ids_add;
    const void *table;
    int64_t table_rows;
    float table_scale;           // on the table's rows
    const int64_t *positions;    // row positions[row] of pos_table is added, or NULL
    const void *pos_table;
    int64_t pos_rows;
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
        const int64_t pos = a.positions ? a.positions[row] : -1;
        const bool placed = pos >= 0 && pos < a.pos_rows;
        const T *psrc = reinterpret_cast<const T *>(a.pos_table) + (placed ? pos : 0) * a.width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            float p[V];
            row_zero<V>(p);
            if (placed && c < a.width) row_load<T, V>(psrc + c, p);
#pragma unroll
            for (int j = 0; j < V; ++j) x[i][j] = fmaf(x[i][j], a.table_scale, p[j]);
        }
    }
    if (a.ids && a.ids_add) {
        const float *src = a.x + row * a.width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            float old[V];
            row_zero<V>(old);
            if (c < a.width) row_load<float, V>(src + c, old);
#pragma unroll
            for (int j = 0; j < V; ++j) x[i][j] += old[j];
        }
    } else if (!a.ids) {
        const float *src = a.x + (have_x ? xrow : 0) * a.width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + lane) * V;
            row_zero<V>(x[i]);
            if (have_x && c < a.width) row_load<float, V>(src + c, x[i]);
        }
    }
    if (a.y) {
        float y[NV][V];
        if (a.mix_w) {
            const float *w = a.mix_w + row * (a.mix + 1);
#pragma unroll
            for (int i = 0; i < NV; ++i) row_zero<V>(y[i]);
            for (int m = 0; m < a.mix + (a.y_extra ? 1 : 0); ++m) {
                const T *src = m < a.mix ? reinterpret_cast<const T *>(a.y) + (row * a.mix + m) * a.width
                                         : reinterpret_cast<const T *>(a.y_extra) + row * a.width;
                const float f = w[m];
#pragma unroll
                for (int i = 0; i < NV; ++i) {
                    const int c = (i * TPR + lane) * V;
                    float t[V];
                    row_zero<V>(t);
                    if (c < a.width) row_load<T, V>(src + c, t);
#pragma unroll
                    for (int j = 0; j < V; ++j) y[i][j] = fmaf(f, t[j], y[i][j]);
                }
            }
        } else {
            const T *src = reinterpret_cast<const T *>(a.y) + row * a.width;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * TPR + lane) * V;
                row_zero<V>(y[i]);
                if (c < a.width) row_load<T, V>(src + c, y[i]);
                if (a.y_bias) {
                    float b[V];
                    row_zero<V>(b);
                    if (c < a.width) row_load<float, V>(a.y_bias + c, b);
#pragma unroll
                    for (int j = 0; j < V; ++j) y[i][j] += b[j];
                }
            }
        }
        if (a.y2) {
            const T *src = reinterpret_cast<const T *>(a.y2) + row * a.width;
            float z[NV][V], sy = 0.f, sz = 0.f;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * TPR + lane) * V;
                row_zero<V>(z[i]);
                if (c < a.width) row_load<T, V>(src + c, z[i]);
#pragma unroll
                for (int j = 0; j < V; ++j) {
                    sy = fmaf(y[i][j], y[i][j], sy);
                    sz = fmaf(z[i][j], z[i][j], sz);
                }
            }
            const float fy = 1.f / sqrtf(row_sum<TPR>(sy, red) / (float)a.width + a.y_eps);
            const float fz = 1.f / sqrtf(row_sum<TPR>(sz, red) / (float)a.width + a.y_eps);
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * TPR + lane) * V;
                float wy[V], wz[V];
                row_zero<V>(wy);
                row_zero<V>(wz);
                if (c < a.width) {
                    row_load<float, V>(a.y_part + c, wy);
                    row_load<float, V>(a.y2_part + c, wz);
                }
#pragma unroll
                for (int j = 0; j < V; ++j) y[i][j] = fmaf(y[i][j] * fy, wy[j], z[i][j] * fz * wz[j]);
            }
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

// ------------------------------------------------------------------ RMS norm + gate
struct RmsGateArgs {
    const void *o;  // [rows][groups * width] of T
    const void *g;  // gate logits, row stride ldg
    int64_t ldg, ldo;
    const float *w;
    void *out;  // row stride ldo
    int64_t rows;  // of one group each: row * groups + group
    int width, groups, gate;
    float eps;
};

template <typename T, int TPR, int V, int NV>
__global__ __launch_bounds__(256) void rms_gate_kernel(const RmsGateArgs a) {
    __shared__ float red[8];
    const int64_t row = (int64_t)blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
    if (row >= a.rows) return;
    const int lane = threadIdx.x % TPR;
    const int64_t trow = a.groups == 1 ? row : row / a.groups;
    const int first = a.groups == 1 ? 0 : (int)(row - trow * a.groups) * a.width;  // column of the group
    const T *src = reinterpret_cast<const T *>(a.o) + row * a.width;
    const T *gate = a.gate == PA_GATE_NONE ? nullptr : reinterpret_cast<const T *>(a.g) + trow * a.ldg + first;
    float x[NV][V], g[NV][V];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        row_zero<V>(x[i]);
        row_zero<V>(g[i]);
        if (c < a.width) {
            row_load<T, V>(src + c, x[i]);
            if (a.gate != PA_GATE_NONE) row_load<T, V>(gate + c, g[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < V; ++j) {
            if (a.gate == PA_GATE_SILU_FIRST) x[i][j] *= row_silu<T>(g[i][j]);
            ss = fmaf(x[i][j], x[i][j], ss);
        }
    const float inv = 1.f / sqrtf(row_sum<TPR>(ss, red) / (float)a.width + a.eps);
    T *dst = reinterpret_cast<T *>(a.out) + trow * a.ldo + first;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (i * TPR + lane) * V;
        if (c >= a.width) continue;
        float w[V], o[V];
        row_load<float, V>(a.w + first + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) {
            o[j] = x[i][j] * inv * w[j];
            if (a.gate == PA_GATE_SIGMOID_LAST) o[j] *= row_sigmoid<T>(g[i][j]);
            if (a.gate == PA_GATE_SILU_LAST) o[j] *= row_silu<T>(g[i][j]);
        }
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
    void *out;  // rows of heads * vdim, row stride ldo
    int64_t ldo;
    int64_t rows;
    int heads, d, vdim;
    float scale;
};

// out = scale * o * sigmoid(gate of the head), the first vdim of every head's d values, packed
template <typename T, int V> __global__ __launch_bounds__(256) void head_gate_kernel(const HeadGateArgs a) {
    const int per_head = a.vdim / V, per_row = a.heads * per_head;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t row = i / per_row;
    if (row >= a.rows) return;
    const int r = (int)(i - row * per_row), h = r / per_head, c = (r - h * per_head) * V;
    float o[V];
    row_load<T, V>(reinterpret_cast<const T *>(a.o) + (row * a.heads + h) * a.d + c, o);
    if (a.g || a.scale != 1.f) {
        float s = a.scale;
        if (a.g) s *= row_sigmoid<T>(pa_scalar<T>::load(reinterpret_cast<const T *>(a.g) + row * a.ldg + h));
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] *= s;
    }
    row_store<T, V>(reinterpret_cast<T *>(a.out) + row * a.ldo + h * a.vdim + c, o);
}

struct BiasActArgs {
    const void *x;  // row stride ldx
    int64_t ldx;
    const float *bias;  // [width], or NULL
    void *out;          // [rows][width]
    int64_t rows;
    int width, act;
};

// out = act(x + bias)
template <typename T, int V> __global__ __launch_bounds__(256) void bias_act_kernel(const BiasActArgs a) {
    const int per_row = (a.width + V - 1) / V;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, row = i / per_row;
    if (row >= a.rows) return;
    const int c = (int)(i - row * per_row) * V;
    float x[V], b[V];
    row_load<T, V>(reinterpret_cast<const T *>(a.x) + row * a.ldx + c, x);
    row_zero<V>(b);
    if (a.bias) {
        if constexpr (V == 8) {
            row_load<float, 4>(a.bias + c, b);
            row_load<float, 4>(a.bias + c + 4, b + 4);
        } else {
            row_load<float, V>(a.bias + c, b);
        }
    }
#pragma unroll
    for (int j = 0; j < V; ++j) {
        const float z = x[j] + b[j], r = fmaxf(z, 0.f);
        x[j] = a.act == PA_ACT_RELU2 ? r * r : a.act == PA_ACT_SILU ? row_silu<T>(z) : a.act == PA_ACT_GELU_TANH ? row_gelu_tanh<T>(z) : z;
    }
    row_store<T, V>(reinterpret_cast<T *>(a.out) + row * a.width + c, x);
}

// out = cap * tanh(x / cap)
template <typename T, int V> __global__ __launch_bounds__(256) void softcap_kernel(const void *x, float *out, int64_t n, float cap) {
    const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (i >= n) return;
    float f[V];
    row_load<T, V>(reinterpret_cast<const T *>(x) + i, f);
#pragma unroll
    for (int j = 0; j < V; ++j) {
        const float z = f[j] / cap;
        f[j] = cap * (sizeof(T) == 4 ? tanhf(z) : 2.f * row_sigmoid<T>(2.f * z) - 1.f);
    }
    row_store<float, V>(out + i, f);
}

// Threads per row and registers per thread by row width: part of a wave, a wave (256 columns), a workgroup.
#define ROW_DISPATCH(KERNEL, T, vec4, width, rows, args, s)                                                \
    do {                                                                                                   \
        const unsigned grid64_ = (unsigned)(((rows) + 3) / 4), grid256_ = (unsigned)(rows);                \
        if (!(vec4)) KERNEL<T, 256, 1, 64><<<dim3(grid256_), dim3(256), 0, s>>>(args);                     \
        else if ((width) <= 64) KERNEL<T, 16, 4, 1><<<dim3((unsigned)(((rows) + 15) / 16)), dim3(256), 0, s>>>(args); \
        else if ((width) <= 128) KERNEL<T, 32, 4, 1><<<dim3((unsigned)(((rows) + 7) / 8)), dim3(256), 0, s>>>(args); \
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

extern "C" int pa_residual_norm(float *x, const void *y, const float *mix_weight, int mix, const void *y_extra,
                                const float *y_bias, const void *y2, const float *y_part, const float *y2_part,
                                const float *y_weight, float y_eps, const int64_t *ids, int ids_add, const void *table,
                                int64_t table_rows, float table_scale, const int64_t *positions, const void *pos_table,
                                int64_t pos_rows, const int64_t *row_index, int64_t x_rows,
                                const float *norm_weight, const float *norm_bias, float eps, int norm, void *out,
                                int64_t rows, int width, int dtype, void *stream) {
    pa_clear_error();
    if (int rc = check_rows("pa_residual_norm", rows, width, dtype)) return rc;
    PA_REQUIRE(norm == PA_NORM_NONE || norm == PA_NORM_LAYER || norm == PA_NORM_RMS, "norm=%d is unknown", norm);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x || ids, "neither a residual nor an embedding to start from");
    PA_REQUIRE(!ids || table, "ids without a table");
    PA_REQUIRE(!row_index || (x && !y && !ids), "row_index only reads the residual");
    PA_REQUIRE(!ids_add || (x && ids), "ids_add without a residual or ids");
    PA_REQUIRE(!y_bias || (y && !mix_weight), "y_bias without a plain y");
    PA_REQUIRE(!y2 || (y && !mix_weight), "y2 without a plain y");
    PA_REQUIRE((y2 != nullptr) == (y_part != nullptr) && (y2 != nullptr) == (y2_part != nullptr), "y2, y_part and y2_part come together");
    PA_REQUIRE(!y_weight || y, "y_weight without y");
    PA_REQUIRE(!positions || (ids && pos_table), "positions without ids or a table");
    PA_REQUIRE(!mix_weight || (y && mix > 0), "mix_weight without y");
    PA_REQUIRE(!y_extra || mix_weight, "y_extra without mix_weight");
    PA_REQUIRE(out || (x && (y || ids)), "nothing to write");
    PA_REQUIRE(norm != PA_NORM_NONE || (!norm_weight && !norm_bias), "norm weights without a norm");
    ResidualArgs a{};
    a.x = x; a.y = y; a.mix_w = mix_weight; a.y_extra = y_extra; a.mix = mix; a.y_weight = y_weight; a.ids = ids;
    a.y_bias = y_bias; a.y2 = y2; a.y_part = y_part; a.y2_part = y2_part; a.ids_add = ids_add;
    a.table = table; a.table_rows = table_rows; a.table_scale = table_scale; a.positions = positions;
    a.pos_table = pos_table; a.pos_rows = pos_rows; a.row_index = row_index; a.x_rows = x_rows; a.w = norm_weight;
    a.b = norm_bias; a.out = out; a.rows = rows; a.width = width; a.norm = norm; a.y_eps = y_eps; a.eps = eps;
    const bool vec4 = width % 4 == 0 && pa_aligned16(x) && pa_aligned16(y) && pa_aligned16(table) && pa_aligned16(out) &&
                      pa_aligned16(y_extra) && pa_aligned16(pos_table) && pa_aligned16(y_bias) && pa_aligned16(y2) &&
                      pa_aligned16(y_part) && pa_aligned16(y2_part) &&
                      pa_aligned16(y_weight) && pa_aligned16(norm_weight) && pa_aligned16(norm_bias);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) ROW_DISPATCH(residual_norm_kernel, float, vec4, width, rows, a, s);
    else ROW_DISPATCH(residual_norm_kernel, pa_bf16, vec4, width, rows, a, s);
    PA_CHECK_LAUNCH("pa_residual_norm");
    return PA_OK;
}

extern "C" int pa_rms_gate(const void *o, const void *gate, int64_t gate_stride, const float *weight, float eps, void *out,
                           int64_t out_stride, int64_t rows, int width, int groups, int gate_mode, int dtype,
                           void *stream) {
    pa_clear_error();
    PA_REQUIRE(groups > 0 && width % groups == 0, "pa_rms_gate: width=%d is not %d equal groups", width, groups);
    const int per = width / groups;
    const int64_t parts = rows * groups;
    if (int rc = check_rows("pa_rms_gate", rows < 0 ? rows : parts, per, dtype)) return rc;
    PA_REQUIRE(gate_mode >= PA_GATE_SIGMOID_LAST && gate_mode <= PA_GATE_NONE, "gate_mode=%d is unknown", gate_mode);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(o && (gate || gate_mode == PA_GATE_NONE) && weight && out, "NULL argument");
    if (gate_mode == PA_GATE_NONE) { gate = nullptr; gate_stride = width; }
    PA_REQUIRE(gate_stride >= width, "gate_stride=%lld is shorter than a row", (long long)gate_stride);
    PA_REQUIRE(out_stride >= width, "out_stride=%lld is shorter than a row", (long long)out_stride);
    RmsGateArgs a{o, gate, gate_stride, out_stride, weight, out, parts, per, groups, gate_mode, eps};
    const uintptr_t four = dtype == PA_F32 ? 15u : 7u;  // four elements
    const bool vec4 = per % 4 == 0 && (gate_mode == PA_GATE_NONE || gate_stride % 4 == 0) && out_stride % 4 == 0 && ((uintptr_t)gate & four) == 0 &&
                      ((uintptr_t)out & four) == 0 && pa_aligned16(o) && pa_aligned16(weight);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) ROW_DISPATCH(rms_gate_kernel, float, vec4, per, parts, a, s);
    else ROW_DISPATCH(rms_gate_kernel, pa_bf16, vec4, per, parts, a, s);
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

extern "C" int pa_bias_act(const void *x, int64_t x_stride, const float *bias, void *out, int64_t rows, int width, int act,
                           int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && width > 0, "pa_bias_act: rows=%lld / width=%d out of range", (long long)rows, width);
    PA_REQUIRE(act >= PA_ACT_SILU && act <= PA_ACT_RELU2, "act=%d is unknown", act);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_bias_act: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(x && out, "NULL argument");
    PA_REQUIRE(x_stride >= width, "x_stride=%lld is shorter than a row", (long long)x_stride);
    BiasActArgs a{x, x_stride, bias, out, rows, width, act};
    const int n = dtype == PA_F32 ? 4 : 8;
    const bool vec = width % n == 0 && x_stride % n == 0 && pa_aligned16(x) && pa_aligned16(bias) && pa_aligned16(out);
    const int64_t items = rows * (vec ? width / n : width), grid = (items + 255) / 256;
    PA_REQUIRE(grid <= 0x7fffffff, "pa_bias_act: rows=%lld is too large for one launch", (long long)rows);
    const dim3 g((unsigned)grid), blk(256);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) {
        if (vec) bias_act_kernel<float, 4><<<g, blk, 0, s>>>(a);
        else bias_act_kernel<float, 1><<<g, blk, 0, s>>>(a);
    } else {
        if (vec) bias_act_kernel<pa_bf16, 8><<<g, blk, 0, s>>>(a);
        else bias_act_kernel<pa_bf16, 1><<<g, blk, 0, s>>>(a);
    }
    PA_CHECK_LAUNCH("pa_bias_act");
    return PA_OK;
}

extern "C" int pa_head_gate(const void *o, const void *gate, int64_t gate_stride, float scale, void *out,
                            int64_t out_stride, int64_t rows, int heads, int d, int vdim, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(rows >= 0 && heads > 0 && d > 0 && vdim > 0 && vdim <= d, "pa_head_gate: sizes out of range");
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_head_gate: dtype=%d is not F32 or BF16", dtype);
    if (rows == 0) return PA_OK;
    PA_REQUIRE(o && out, "NULL argument");
    PA_REQUIRE(!gate || gate_stride >= heads, "gate_stride=%lld is shorter than a row", (long long)gate_stride);
    PA_REQUIRE(out_stride >= (int64_t)heads * vdim, "out_stride=%lld is shorter than a row", (long long)out_stride);
    HeadGateArgs a{o, gate, gate_stride, out, out_stride, rows, heads, d, vdim, scale};
    const int n = dtype == PA_F32 ? 4 : 8;
    const bool vec = d % n == 0 && vdim % n == 0 && out_stride % n == 0 && pa_aligned16(o) && pa_aligned16(out);
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

extern "C" int pa_softcap(const void *x, float *out, int64_t n, float cap, int dtype, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n >= 0 && cap > 0.f, "pa_softcap: n / cap out of range");
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_softcap: dtype=%d is not F32 or BF16", dtype);
    if (n == 0) return PA_OK;
    PA_REQUIRE(x && out, "NULL argument");
    const bool vec = n % 4 == 0 && pa_aligned16(x) && pa_aligned16(out);
    const int64_t grid = ((vec ? n / 4 : n) + 255) / 256;
    PA_REQUIRE(grid <= 0x7fffffff, "pa_softcap: n=%lld is too large for one launch", (long long)n);
    const dim3 g((unsigned)grid), blk(256);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PA_F32) {
        if (vec) softcap_kernel<float, 4><<<g, blk, 0, s>>>(x, out, n, cap);
        else softcap_kernel<float, 1><<<g, blk, 0, s>>>(x, out, n, cap);
    } else {
        if (vec) softcap_kernel<pa_bf16, 4><<<g, blk, 0, s>>>(x, out, n, cap);
        else softcap_kernel<pa_bf16, 1><<<g, blk, 0, s>>>(x, out, n, cap);
    }
    PA_CHECK_LAUNCH("pa_softcap");
    return PA_OK;
}
