// Entry points of attention with score terms, and its kernel on the vector units: 32-bit rows, and sizes that the matrix-core
// kernels (scored_decode.hip, scored_prefill.hip) do not have.
#include "scored_attn.h"

namespace {

// A wave per (row, head).  A lane scores one key at a time, 64 keys side by side; then the lanes turn to the value columns.
template <typename T, int VPL> __global__ __launch_bounds__(256) void scored_vector_kernel(const ScoredArgs a) {
    extern __shared__ float scored_lds[];
    const int b = blockIdx.z, i = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x / 64, h = blockIdx.x * 4 + wave;
    ScoredPortion p;
    if (h >= a.heads || !scored_portion(a, b, p) || i >= p.n) return;
    const int64_t row = p.row0 + i;
    const int pos = p.pos0 + i, n = a.n1 + a.n2;
    float *q = scored_lds + wave * n;
    const T *q1 = reinterpret_cast<const T *>(a.q1) + row * a.q1_row + h * a.q1_head;
    const T *q2 = reinterpret_cast<const T *>(a.q2) + row * a.q2_row + h * a.q2_head;
    for (int e = lane; e < n; e += 64) q[e] = pa_scalar<T>::load(e < a.n1 ? q1 + e : q2 + (e - a.n1));
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");  // (a wave's own part of LDS)
    __builtin_amdgcn_wave_barrier();
    const int32_t *table = a.bt + b * a.bt_stride;
    const int kvh = h / a.n_rep;
    const T *k = reinterpret_cast<const T *>(a.k) + (int64_t)kvh * a.k_dim, *v = reinterpret_cast<const T *>(a.v) + (int64_t)kvh * a.v_dim;
    float m = a.sink ? a.sink[h] : kScoredNone, l = a.sink ? 1.f : 0.f;
    float acc[VPL];
    row_zero<VPL>(acc);
    for (int j0 = scored_first_key(a, pos); j0 <= pos; j0 += 64) {
        const int j = j0 + lane;
        const int64_t slot = j <= pos ? scored_slot(a, table, j) : -1;
        float s = 0.f;
        if (slot >= 0) {
            const T *kr = k + slot * ((int64_t)a.hkv * a.k_dim);
            for (int e = 0; e < n; ++e) s = fmaf(q[e], pa_scalar<T>::load(kr + e), s);
        }
        s *= a.scale;
        if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
        if (a.bias && j <= pos) s += a.bias[(int64_t)h * a.bias_n + (pos - j < a.bias_n ? pos - j : a.bias_n - 1)];
        if (j > pos) s = kScoredNone;
        float top = s;
#pragma unroll
        for (int d = 32; d > 0; d /= 2) top = fmaxf(top, __shfl_xor(top, d, 64));
        const float next = fmaxf(m, top), keep = expf(m - next);
        m = next;
        const float w = j <= pos ? expf(s - m) : 0.f;
        l = l * keep + pa_group_sum<64>(w);
#pragma unroll
        for (int c = 0; c < VPL; ++c) acc[c] *= keep;
        const int keys = pos - j0 + 1 < 64 ? pos - j0 + 1 : 64;
        for (int t = 0; t < keys; ++t) {
            const int64_t at = __shfl(slot, t, 64);
            const float f = __shfl(w, t, 64);
            if (at < 0) continue;
            const T *vr = v + at * ((int64_t)a.hkv * a.v_dim);
#pragma unroll
            for (int c = 0; c < VPL; ++c)
                if (c * 64 + lane < a.vdim) acc[c] = fmaf(f, pa_scalar<T>::load(vr + c * 64 + lane), acc[c]);
        }
    }
    T *out = reinterpret_cast<T *>(a.out) + (row * a.heads + h) * a.vdim;
#pragma unroll
    for (int c = 0; c < VPL; ++c)
        if (c * 64 + lane < a.vdim) pa_scalar<T>::store(out + c * 64 + lane, acc[c] / l);
}

template <typename T> void launch_vector(const ScoredArgs &a, hipStream_t s) {
    const dim3 grid((unsigned)((a.heads + 3) / 4), (unsigned)a.max_q_len, (unsigned)a.batch), block(256);
    const size_t lds = (size_t)4 * (a.n1 + a.n2) * sizeof(float);
    if (a.vdim <= 256) scored_vector_kernel<T, 4><<<grid, block, lds, s>>>(a);
    else scored_vector_kernel<T, 16><<<grid, block, lds, s>>>(a);
}

int scored_cus() {
    static int cached[64];
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return 256;
    int n = __atomic_load_n(&cached[dev], __ATOMIC_RELAXED);
    if (n == 0) {
        if (hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0) n = 256;
        __atomic_store_n(&cached[dev], n, __ATOMIC_RELAXED);
    }
    return n;
}

int plan_splits(int batch, int heads, int hkv, bool one, int vc, int64_t max_keys, int window) {
    const int rep = heads / hkv, tile = one && rep > 32 ? 64 : one && rep > 16 ? 32 : 16;
    const int64_t workgroups = (int64_t)batch * hkv * ((rep + tile - 1) / tile);
    return scored_splits(workgroups, scored_cus(), window > 0 && window < max_keys ? window : max_keys, vc > 256);
}

}  // namespace

extern "C" size_t pa_scored_workspace_bytes(int batch, int num_q_heads, int num_kv_heads, int key_size, int vdim, int one_tensor,
                                            int64_t max_keys, int window) {
    if (batch <= 0 || num_kv_heads <= 0 || num_q_heads <= 0) return 0;
    const int vc = scored_value_cols(key_size, vdim, one_tensor != 0);
    const int splits = plan_splits(batch, num_q_heads, num_kv_heads, one_tensor != 0, vc, max_keys, window);
    return splits > 1 && vc ? (size_t)batch * num_q_heads * splits * (vc + 2) * sizeof(float) : 0;
}

extern "C" int pa_scored_attention(const void *q1, int64_t q1_row, int64_t q1_head, int n1, const void *q2, int64_t q2_row,
                                   int64_t q2_head, int n2, const void *k_cache, int k_dim, const void *v_cache, int v_dim, int vdim,
                                   const int32_t *block_tables, int64_t bt_stride, int block_size, int64_t num_blocks,
                                   const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts, int64_t n_rows, int batch,
                                   int max_q_len, int num_q_heads, int num_kv_heads, float scale, int window, float softcap,
                                   const float *bias, int bias_n, const float *sink, void *out, int dtype, void *workspace,
                                   size_t workspace_bytes, void *stream) {
    pa_clear_error();
    PA_REQUIRE(n_rows >= 0 && batch >= 0 && max_q_len >= 0 && num_blocks >= 0 && bt_stride >= 0, "pa_scored_attention: a count is negative");
    PA_REQUIRE(n1 > 0 && n2 >= 0 && vdim > 0 && k_dim >= n1 + n2 && v_dim >= vdim, "pa_scored_attention: n1 / n2 / vdim do not fit the pool");
    PA_REQUIRE(num_q_heads > 0 && num_kv_heads > 0 && num_q_heads % num_kv_heads == 0,
               "num_q_heads=%d must be a positive multiple of num_kv_heads=%d", num_q_heads, num_kv_heads);
    PA_REQUIRE(block_size > 0 && window >= 0, "block_size=%d / window=%d out of range", block_size, window);
    PA_REQUIRE(softcap >= 0.f && (!bias || bias_n > 0), "softcap / bias_n out of range");
    PA_REQUIRE((q_lens == nullptr) == (q_starts == nullptr), "q_lens and q_starts come together");
    PA_REQUIRE(batch <= 65535 && max_q_len <= 65535, "batch=%d / max_q_len=%d above 65535", batch, max_q_len);
    if (dtype != PA_F32 && dtype != PA_BF16) return pa_fail(PA_ERR_UNSUPPORTED, "pa_scored_attention: dtype=%d is not F32 or BF16", dtype);
    if (vdim > 1024 || n1 + n2 > 2048)
        return pa_fail(PA_ERR_UNSUPPORTED, "pa_scored_attention: value size %d above 1024 or key size %d above 2048", vdim, n1 + n2);
    if (n_rows == 0 || batch == 0 || (q_lens && max_q_len == 0)) return PA_OK;
    PA_REQUIRE(q1 && (q2 || n2 == 0) && k_cache && v_cache && ctx_lens && out && (block_tables || bt_stride == 0),
               "pa_scored_attention: NULL argument");
    PA_REQUIRE(q_lens || n_rows >= batch, "n_rows=%lld below batch=%d", (long long)n_rows, batch);
    ScoredArgs a{};
    a.q1 = q1; a.q1_row = q1_row; a.q1_head = q1_head; a.n1 = n1;
    a.q2 = q2 ? q2 : q1; a.q2_row = q2_row; a.q2_head = q2_head; a.n2 = n2;
    a.k = k_cache; a.v = v_cache; a.k_dim = k_dim; a.v_dim = v_dim; a.vdim = vdim;
    a.bt = block_tables; a.bt_stride = bt_stride; a.num_blocks = num_blocks; a.bs = block_size;
    a.ctx_lens = ctx_lens; a.q_lens = q_lens; a.q_starts = q_starts; a.n_rows = n_rows; a.batch = batch;
    a.max_q_len = q_lens ? max_q_len : 1; a.heads = num_q_heads; a.hkv = num_kv_heads; a.n_rep = num_q_heads / num_kv_heads;
    a.window = window; a.scale = scale; a.cap = softcap; a.bias = bias; a.bias_n = bias_n; a.sink = sink; a.out = out;
    a.splits = 1;
    hipStream_t s = (hipStream_t)stream;
    const bool one = k_cache == v_cache;
    if (!q_lens && workspace) {
        const int vc = scored_value_cols(n1 + n2, vdim, one);
        a.splits = plan_splits(batch, num_q_heads, num_kv_heads, one, vc, bt_stride * block_size, window);
        const size_t per = (size_t)batch * num_q_heads * (vc + 2) * sizeof(float);
        while (a.splits > 1 && per * a.splits > workspace_bytes) --a.splits;
        a.part_o = (float *)workspace;
        a.part_ml = a.part_o + (size_t)batch * num_q_heads * a.splits * vc;
        PA_REQUIRE(a.splits == 1 || pa_aligned16(workspace), "the workspace must be 16-byte aligned");
    }
    int rc = PA_OK;
    if (pa_scored_decode_launch(a, dtype, s, rc) || pa_scored_prefill_launch(a, dtype, s, rc)) return rc;
    if (dtype == PA_F32) launch_vector<float>(a, s);
    else launch_vector<pa_bf16>(a, s);
    PA_CHECK_LAUNCH("pa_scored_attention");
    return PA_OK;
}
