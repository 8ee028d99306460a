// serve_rows.hip -- one-workgroup-per-token kernels of the serving engine: embedding, fused residual + layer norm, the
// latent projections' norms + rotary + cache write, the latent query, the output gate.  Statistics and angles are float.
#include "serve_common.h"

static thread_local char g_err[512] = "";
void qsv_set_error(const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
}
extern "C" int qsv_version(void) { return 1; }
extern "C" const char* qsv_arch(void) { return "gfx950"; }
extern "C" const char* qsv_last_error(void) { return g_err; }

constexpr int NT = 256;

// ---- embedding ---------------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(NT) void embed_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ table,
                                                   const int32_t* __restrict__ tokens, int D) {
    const size_t t = blockIdx.x;
    const T* row = table + (size_t)tokens[t] * D;
    for (int i = threadIdx.x; i < D; i += NT) {
        const float v = ld(row, i);
        x[t * D + i] = v;
        st(h, t * D + i, v);
    }
}
extern "C" int qsv_embed(float* x, void* h, const void* table, const int32_t* tokens, int n, int D, int dtype, void* stream) {
    QSV_REQUIRE(x && h && table && tokens && n >= 0 && D > 0, "qsv_embed: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_embed",
                 hipLaunchKernelGGL(embed_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)table, tokens, D));
    return qsv_launch_status("qsv_embed");
}

// ---- x += layer_norm(y) * w ; h = x -------------------------------------------------------------------------------------------
// Two reductions (mean, then the mean of squared deviations); the row of y is re-read from cache, not held in registers, so any
// width works.
template <typename T>
__global__ __launch_bounds__(NT) void add_layer_norm_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ y,
                                                            const T* __restrict__ w, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    const T* yr = y + t * D;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) s += ld(yr, i);
    const float mean = block_sum<NT>(s, red) / (float)D;
    float q = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) {
        const float d = ld(yr, i) - mean;
        q += d * d;
    }
    const float inv = 1.0f / sqrtf(block_sum<NT>(q, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) {
        const float v = x[t * D + i] + (ld(yr, i) - mean) * inv * ld(w, i);
        x[t * D + i] = v;
        st(h, t * D + i, v);
    }
}
extern "C" int qsv_add_layer_norm(float* x, void* h, const void* y, const void* w, float eps, int n, int D, int dtype,
                                  void* stream) {
    QSV_REQUIRE(x && h && y && w && n >= 0 && D > 0, "qsv_add_layer_norm: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_add_layer_norm",
                 hipLaunchKernelGGL(add_layer_norm_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)y,
                                    (const T*)w, eps, D));
    return qsv_launch_status("qsv_add_layer_norm");
}

template <typename T>
__global__ __launch_bounds__(NT) void layer_norm_rows_kernel(T* __restrict__ out, const float* __restrict__ x,
                                                             const int32_t* __restrict__ rows, const T* __restrict__ w,
                                                             float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t r = blockIdx.x;
    const float* xr = x + (size_t)(rows ? rows[r] : (int32_t)r) * D;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) s += xr[i];
    const float mean = block_sum<NT>(s, red) / (float)D;
    float q = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) {
        const float d = xr[i] - mean;
        q += d * d;
    }
    const float inv = 1.0f / sqrtf(block_sum<NT>(q, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) st(out, r * D + i, (xr[i] - mean) * inv * ld(w, i));
}
extern "C" int qsv_layer_norm_rows(void* out, const float* x, const int32_t* rows, const void* w, float eps, int n, int D,
                                   int dtype, void* stream) {
    QSV_REQUIRE(out && x && w && n >= 0 && D > 0, "qsv_layer_norm_rows: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_layer_norm_rows",
                 hipLaunchKernelGGL(layer_norm_rows_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, (T*)out, x, rows,
                                    (const T*)w, eps, D));
    return qsv_launch_status("qsv_layer_norm_rows");
}

// ---- latent projections: two RMS norms, the rotary key part, the cache row ---------------------------------------------------
template <typename T>
__global__ __launch_bounds__(NT) void latent_prep_kernel(const T* __restrict__ down, int64_t down_stride, int q_off, int q_rank,
                                                         const T* __restrict__ q_w, T* __restrict__ cq, int kv_off, int kv_rank,
                                                         const T* __restrict__ kv_w, int rot_dim, int rot_n,
                                                         const float* __restrict__ rope, T* __restrict__ pool,
                                                         const int64_t* __restrict__ slot, const int32_t* __restrict__ pos,
                                                         float eps) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    const T* row = down + t * down_stride;
    float s = 0.f;
    for (int i = threadIdx.x; i < q_rank; i += NT) {
        const float v = ld(row, q_off + i);
        s += v * v;
    }
    const float qinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)q_rank + eps);
    for (int i = threadIdx.x; i < q_rank; i += NT) st(cq, t * q_rank + i, ld(row, q_off + i) * qinv * ld(q_w, i));
    s = 0.f;
    for (int i = threadIdx.x; i < kv_rank; i += NT) {
        const float v = ld(row, kv_off + i);
        s += v * v;
    }
    const float kinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)kv_rank + eps);
    T* dst = pool + (size_t)slot[t] * (size_t)(kv_rank + rot_dim);
    for (int i = threadIdx.x; i < kv_rank; i += NT) st(dst, i, ld(row, kv_off + i) * kinv * ld(kv_w, i));
    const int half = rot_n / 2;
    const float* cs = rope ? rope + (size_t)pos[t] * (size_t)rot_n : nullptr;   // [2, half]: cos then sin
    const T* kr = row + kv_off + kv_rank;
    for (int i = threadIdx.x; i < rot_dim; i += NT) {
        float v = ld(kr, i);
        if (i < rot_n) {
            const int p = i >> 1;
            const float c = cs[p], sn = cs[half + p];
            const float u = ld(kr, 2 * p), w2 = ld(kr, 2 * p + 1);
            v = (i & 1) ? (w2 * c + u * sn) : (u * c - w2 * sn);
        }
        st(dst, kv_rank + i, v);
    }
}
extern "C" int qsv_latent_prep(const void* down, int64_t down_stride, int q_off, int q_rank, const void* q_w, void* cq,
                               int kv_off, int kv_rank, const void* kv_w, int rot_dim, int rot_n, const float* rope,
                               void* pool, const int64_t* slot, const int32_t* pos, float eps, int n, int dtype, void* stream) {
    QSV_REQUIRE(down && q_w && cq && kv_w && pool && slot && pos && n >= 0, "qsv_latent_prep: null argument");
    QSV_REQUIRE(q_rank > 0 && kv_rank > 0 && rot_dim >= 0 && rot_n >= 0 && rot_n <= rot_dim && rot_n % 2 == 0,
                "qsv_latent_prep: bad sizes (q_rank %d, kv_rank %d, rot_dim %d, rotated %d)", q_rank, kv_rank, rot_dim, rot_n);
    QSV_REQUIRE(rot_n == 0 || rope, "qsv_latent_prep: rotary part without a cos / sin table");
    QSV_REQUIRE(q_off >= 0 && kv_off >= 0 && q_off + q_rank <= down_stride && kv_off + kv_rank + rot_dim <= down_stride,
                "qsv_latent_prep: the slices do not fit a row of %lld elements", (long long)down_stride);
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_latent_prep",
                 hipLaunchKernelGGL(latent_prep_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, (const T*)down, down_stride,
                                    q_off, q_rank, (const T*)q_w, (T*)cq, kv_off, kv_rank, (const T*)kv_w, rot_dim, rot_n, rope,
                                    (T*)pool, slot, pos, eps));
    return qsv_launch_status("qsv_latent_prep");
}

// ---- the query in the latent space: [absorbed part | rotated part], scaled, float ---------------------------------------------
// One workgroup per token, all heads: the absorbed part is a strided gather ([H, T, rank] -> [T, H, rank + rot]), the rotated
// part a handful of values per head.
template <typename T>
__global__ __launch_bounds__(NT) void latent_query_kernel(float* __restrict__ qf, const T* __restrict__ q,
                                                          const T* __restrict__ q_abs, const float* __restrict__ rope,
                                                          const int32_t* __restrict__ pos, float scale, int n_tokens, int H,
                                                          int dim, int rot_dim, int rot_n, int rank) {
    const size_t t = blockIdx.x;
    const int R = rank + rot_dim;
    float* dst = qf + t * H * (size_t)R;
    for (int i = threadIdx.x; i < H * rank; i += NT) {
        const int h = i / rank, c = i - h * rank;
        dst[(size_t)h * R + c] = ld(q_abs, ((size_t)h * n_tokens + t) * (size_t)rank + c) * scale;
    }
    const int half = rot_n / 2;
    const float* cs = rope ? rope + (size_t)pos[t] * (size_t)rot_n : nullptr;
    for (int i = threadIdx.x; i < H * rot_dim; i += NT) {
        const int h = i / rot_dim, c = i - h * rot_dim;
        const T* qr = q + (t * H + h) * (size_t)(dim + rot_dim) + dim;
        float v = ld(qr, c);
        if (c < rot_n) {
            const int p = c >> 1;
            const float co = cs[p], sn = cs[half + p];
            const float u = ld(qr, 2 * p), w2 = ld(qr, 2 * p + 1);
            v = (c & 1) ? (w2 * co + u * sn) : (u * co - w2 * sn);
        }
        dst[(size_t)h * R + rank + c] = v * scale;
    }
}
extern "C" int qsv_latent_query(float* qf, const void* q, const void* q_abs, const float* rope, const int32_t* pos, float scale,
                                int n, int H, int dim, int rot_dim, int rot_n, int rank, int dtype, void* stream) {
    QSV_REQUIRE(qf && q && q_abs && pos && n >= 0 && H > 0 && dim > 0 && rank > 0, "qsv_latent_query: bad arguments");
    QSV_REQUIRE(rot_dim >= 0 && rot_n >= 0 && rot_n <= rot_dim && rot_n % 2 == 0 && (rot_n == 0 || rope),
                "qsv_latent_query: bad rotary sizes (%d of %d)", rot_n, rot_dim);
    if (n == 0) return QSV_OK;
    QSV_REQUIRE((int64_t)n * H < (1ll << 31), "qsv_latent_query: too many (token, head) pairs");
    QSV_DISPATCH(dtype, "qsv_latent_query",
                 hipLaunchKernelGGL(latent_query_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, qf, (const T*)q,
                                    (const T*)q_abs, rope, pos, scale, n, H, dim, rot_dim, rot_n, rank));
    return qsv_launch_status("qsv_latent_query");
}

// ---- output gate ---------------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(NT) void sigmoid_gate_kernel(T* __restrict__ o, const T* __restrict__ g, int64_t g_stride, int n) {
    const size_t t = blockIdx.x;
    for (int i = threadIdx.x; i < n; i += NT) {
        const float gate = 1.0f / (1.0f + expf(-ld(g, t * g_stride + i)));
        st(o, t * n + i, ld(o, t * n + i) * gate);
    }
}
extern "C" int qsv_sigmoid_gate(void* o, const void* g, int64_t g_stride, int n_tokens, int n, int dtype, void* stream) {
    QSV_REQUIRE(o && g && n_tokens >= 0 && n > 0 && g_stride >= n, "qsv_sigmoid_gate: bad arguments");
    if (n_tokens == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_sigmoid_gate",
                 hipLaunchKernelGGL(sigmoid_gate_kernel<T>, dim3(n_tokens), dim3(NT), 0, (hipStream_t)stream, (T*)o, (const T*)g,
                                    g_stride, n));
    return qsv_launch_status("qsv_sigmoid_gate");
}

// ---- embedding with a sinusoidal position vector ---------------------------------------------------------------------------------
// x[t, 2i] = table[tok, 2i] * scale + sin(pos * freq[i]),  x[t, 2i + 1] = ... + cos(pos * freq[i]); the angle is a float product.
template <typename T>
__global__ __launch_bounds__(NT) void embed_sinusoid_kernel(float* __restrict__ x, const T* __restrict__ table,
                                                            const int32_t* __restrict__ tokens, const int32_t* __restrict__ pos,
                                                            const float* __restrict__ freq, float scale, int D) {
    const size_t t = blockIdx.x;
    const T* row = table + (size_t)tokens[t] * D;
    const float p = (float)pos[t];
    for (int i = threadIdx.x; i < D; i += NT) {
        const float a = p * freq[i >> 1];
        x[t * D + i] = ld(row, i) * scale + ((i & 1) ? cosf(a) : sinf(a));
    }
}
extern "C" int qsv_embed_sinusoid(float* x, const void* table, const int32_t* tokens, const int32_t* pos, const float* freq,
                                  float scale, int n, int D, int dtype, void* stream) {
    QSV_REQUIRE(x && table && tokens && pos && freq && n >= 0 && D > 0, "qsv_embed_sinusoid: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_embed_sinusoid",
                 hipLaunchKernelGGL(embed_sinusoid_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (const T*)table, tokens, pos,
                                    freq, scale, D));
    return qsv_launch_status("qsv_embed_sinusoid");
}

// ---- x += a + (b + c); h = rms_norm(x) * w -----------------------------------------------------------------------------------------
// a, b, c: the sublayers' outputs (each may be NULL); h (may be NULL: no norm) is the next layer's input in the storage type.
template <typename T>
__global__ __launch_bounds__(NT) void add_rms_norm_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ a,
                                                          const T* __restrict__ b, const T* __restrict__ c, const T* __restrict__ w,
                                                          float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) {
        float v = x[t * D + i];
        if (a || b || c) {
            float y = 0.f;
            if (b) y = ld(b, t * D + i);
            if (c) y += ld(c, t * D + i);
            if (a) y = ld(a, t * D + i) + y;
            v += y;
            x[t * D + i] = v;
        }
        s += v * v;
    }
    if (!h) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) st(h, t * D + i, x[t * D + i] * inv * ld(w, i));   // (this thread's own writes)
}
// The same for widths that are multiples of four, up to 4 * NT * VPT: 16-byte accesses of the stream (8-byte of bfloat16 rows), the
// row stays in registers between the sum of squares and the scaling.
__device__ __forceinline__ float4 ld4v(const float* p, size_t i) { return *(const float4*)(p + i); }
__device__ __forceinline__ float4 ld4v(const bf16_t* p, size_t i) {
    const uint2 u = *(const uint2*)(p + i);
    return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                       __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ void st4v(float* p, size_t i, float4 v) { *(float4*)(p + i) = v; }
__device__ __forceinline__ void st4v(bf16_t* p, size_t i, float4 v) {
    uint2 u;
    u.x = (uint32_t)f2bf(v.x) | ((uint32_t)f2bf(v.y) << 16);
    u.y = (uint32_t)f2bf(v.z) | ((uint32_t)f2bf(v.w) << 16);
    *(uint2*)(p + i) = u;
}
template <typename T, int VPT>
__global__ __launch_bounds__(NT) void add_rms_norm_vec_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ a,
                                                              const T* __restrict__ b, const T* __restrict__ c,
                                                              const T* __restrict__ w, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float4 v[VPT];
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        v[k] = ld4v(x, t * D + i);
        if (a || b || c) {
            float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
            if (b) y = ld4v(b, t * D + i);
            if (c) {
                const float4 z = ld4v(c, t * D + i);
                y.x += z.x; y.y += z.y; y.z += z.z; y.w += z.w;
            }
            if (a) {
                const float4 z = ld4v(a, t * D + i);
                y.x = z.x + y.x; y.y = z.y + y.y; y.z = z.z + y.z; y.w = z.w + y.w;
            }
            v[k].x += y.x; v[k].y += y.y; v[k].z += y.z; v[k].w += y.w;
            st4v(x, t * D + i, v[k]);
        }
        s += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
    }
    if (!h) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        const float4 g = ld4v(w, i);
        st4v(h, t * D + i, make_float4(v[k].x * inv * g.x, v[k].y * inv * g.y, v[k].z * inv * g.z, v[k].w * inv * g.w));
    }
}
extern "C" int qsv_add_rms_norm(float* x, void* h, const void* a, const void* b, const void* c, const void* w, float eps, int n,
                                int D, int dtype, void* stream) {
    QSV_REQUIRE(x && n >= 0 && D > 0 && (!h || w), "qsv_add_rms_norm: bad arguments");
    if (n == 0) return QSV_OK;
    const int vecs = (D / 4 + NT - 1) / NT;
    if (D % 4 == 0 && vecs <= 8) {
#define QSV_ARN(V)                                                                                                                 \
    QSV_DISPATCH(dtype, "qsv_add_rms_norm",                                                                                        \
                 hipLaunchKernelGGL((add_rms_norm_vec_kernel<T, V>), dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)a, \
                                    (const T*)b, (const T*)c, (const T*)w, eps, D))
        if (vecs <= 1) QSV_ARN(1);
        else if (vecs <= 2) QSV_ARN(2);
        else if (vecs <= 4) QSV_ARN(4);
        else QSV_ARN(8);
#undef QSV_ARN
        return qsv_launch_status("qsv_add_rms_norm");
    }
    QSV_DISPATCH(dtype, "qsv_add_rms_norm",
                 hipLaunchKernelGGL(add_rms_norm_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)a, (const T*)b,
                                    (const T*)c, (const T*)w, eps, D));
    return qsv_launch_status("qsv_add_rms_norm");
}

// ---- x += s0 a + s1 b + s2 c (element-wise scales); h0 = rms_norm(x) * g0, h1 = rms_norm(x) * g1 -------------------------------------------
// The parallel layer with a norm of its own for each side: one statistic, two gains (float, one per coordinate).  tokens: x starts as the
// embedding row.  a, b, c (storage type), their scales and h1 may be NULL; h0 == NULL: the sum only.
struct ScaledParts {
    const void *y[3], *s[3];
};
template <typename T, int VPT>
__global__ __launch_bounds__(NT) void scaled_sum_rms_norms_vec_kernel(float* __restrict__ x, T* __restrict__ h0, T* __restrict__ h1, ScaledParts p,
                                                                      const float* __restrict__ g0, const float* __restrict__ g1,
                                                                      const int32_t* __restrict__ tokens, const T* __restrict__ table, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float4 v[VPT];
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        v[k] = tokens ? ld4v(table, (size_t)tokens[t] * D + i) : ld4v(x, t * D + i);
        float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int j = 0; j < 3; ++j)
            if (p.y[j]) {
                const float4 z = ld4v((const T*)p.y[j], t * D + i);
                const float4 f = p.s[j] ? ld4v((const T*)p.s[j], i) : make_float4(1.f, 1.f, 1.f, 1.f);
                y.x += f.x * z.x; y.y += f.y * z.y; y.z += f.z * z.z; y.w += f.w * z.w;
            }
        v[k].x += y.x; v[k].y += y.y; v[k].z += y.z; v[k].w += y.w;
        st4v(x, t * D + i, v[k]);
        s += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
    }
    if (!h0) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        const float4 n = make_float4(v[k].x * inv, v[k].y * inv, v[k].z * inv, v[k].w * inv);
        const float4 a = ld4v(g0, i);
        st4v(h0, t * D + i, make_float4(n.x * a.x, n.y * a.y, n.z * a.z, n.w * a.w));
        if (h1) {
            const float4 b = ld4v(g1, i);
            st4v(h1, t * D + i, make_float4(n.x * b.x, n.y * b.y, n.z * b.z, n.w * b.w));
        }
    }
}
template <typename T>
__global__ __launch_bounds__(NT) void scaled_sum_rms_norms_kernel(float* __restrict__ x, T* __restrict__ h0, T* __restrict__ h1, ScaledParts p,
                                                                  const float* __restrict__ g0, const float* __restrict__ g1,
                                                                  const int32_t* __restrict__ tokens, const T* __restrict__ table, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) {
        float v = tokens ? ld(table, (size_t)tokens[t] * D + i) : x[t * D + i], y = 0.f;
#pragma unroll
        for (int j = 0; j < 3; ++j)
            if (p.y[j]) y += (p.s[j] ? ld((const T*)p.s[j], i) : 1.f) * ld((const T*)p.y[j], t * D + i);
        v += y;
        x[t * D + i] = v;
        s += v * v;
    }
    if (!h0) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) {
        const float n = x[t * D + i] * inv;              // (this thread's own writes)
        st(h0, t * D + i, n * g0[i]);
        if (h1) st(h1, t * D + i, n * g1[i]);
    }
}
extern "C" int qsv_scaled_sum_rms_norms(float* x, void* h0, void* h1, const void* a, const void* sa, const void* b, const void* sb, const void* c,
                                        const void* sc, const float* g0, const float* g1, const int32_t* tokens, const void* table, float eps,
                                        int n, int D, int dtype, void* stream) {
    QSV_REQUIRE(x && n >= 0 && D > 0 && (!h0 || g0) && (!h1 || (h0 && g1)) && (!tokens || table), "qsv_scaled_sum_rms_norms: bad arguments");
    if (n == 0) return QSV_OK;
    const ScaledParts p = {{a, b, c}, {sa, sb, sc}};
    const int vecs = (D / 4 + NT - 1) / NT;
#define QSV_SSN(V)                                                                                                                 \
    QSV_DISPATCH(dtype, "qsv_scaled_sum_rms_norms",                                                                                \
                 hipLaunchKernelGGL((scaled_sum_rms_norms_vec_kernel<T, V>), dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h0, (T*)h1, p, g0, \
                                    g1, tokens, (const T*)table, eps, D))
    if (D % 4 == 0 && vecs <= 8) {
        if (vecs <= 1) QSV_SSN(1);
        else if (vecs <= 2) QSV_SSN(2);
        else if (vecs <= 4) QSV_SSN(4);
        else QSV_SSN(8);
    } else {
        QSV_DISPATCH(dtype, "qsv_scaled_sum_rms_norms",
                     hipLaunchKernelGGL(scaled_sum_rms_norms_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h0, (T*)h1, p, g0, g1,
                                        tokens, (const T*)table, eps, D));
    }
#undef QSV_SSN
    return qsv_launch_status("qsv_scaled_sum_rms_norms");
}

template <typename T, typename TW>
__global__ __launch_bounds__(NT) void rms_norm_rows_kernel(T* __restrict__ out, const float* __restrict__ x,
                                                           const int32_t* __restrict__ rows, const TW* __restrict__ w, float eps,
                                                           int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t r = blockIdx.x;
    const float* xr = x + (size_t)(rows ? rows[r] : (int32_t)r) * D;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) s += xr[i] * xr[i];
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) st(out, r * D + i, xr[i] * inv * ld(w, i));
}
extern "C" int qsv_rms_norm_rows(void* out, const float* x, const int32_t* rows, const void* w, int w_dtype, float eps, int n, int D,
                                 int dtype, void* stream) {
    QSV_REQUIRE(out && x && w && n >= 0 && D > 0 && (w_dtype == dtype || w_dtype == QSV_F32), "qsv_rms_norm_rows: bad arguments");
    if (n == 0) return QSV_OK;
    if (w_dtype == QSV_F32)
        QSV_DISPATCH(dtype, "qsv_rms_norm_rows",
                     hipLaunchKernelGGL((rms_norm_rows_kernel<T, float>), dim3(n), dim3(NT), 0, (hipStream_t)stream, (T*)out, x, rows,
                                        (const float*)w, eps, D));
    else
        hipLaunchKernelGGL((rms_norm_rows_kernel<bf16_t, bf16_t>), dim3(n), dim3(NT), 0, (hipStream_t)stream, (bf16_t*)out, x, rows,
                           (const bf16_t*)w, eps, D);
    return qsv_launch_status("qsv_rms_norm_rows");
}

// ---- attention with queries and keys normed over all heads at once, and values blended with an earlier layer's ------------------
//   qf[t, h]          = [ 0 (vdim) | rms_norm(q[t])[h] * q_w[h] * scale ]       float [T, heads, vdim + dim]; the norm runs over all
//   pool[g, slot[t]]  = [ v'[t, g] | rms_norm(k[t])[g] * k_w[g] ]               heads * dim (kv_heads * dim) values of the projection
//   v' = (1 - mix) v + mix v_first  where v_first (row stride vf_stride, [kv_heads * vdim] per token) is given, else v.
template <typename T>
__global__ __launch_bounds__(NT) void normed_attention_prep_kernel(float* __restrict__ qf, T* __restrict__ pool, int64_t pool_rows,
                                                                   const T* __restrict__ proj, int64_t stride, int q_off, int k_off,
                                                                   int v_off, int H, int G, int dim, int vdim,
                                                                   const T* __restrict__ q_w, const T* __restrict__ k_w, float eps,
                                                                   float scale, const T* __restrict__ v_first, int64_t vf_stride,
                                                                   float mix, const int64_t* __restrict__ slot) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    const int R = vdim + dim;
    const T* row = proj + t * stride;
    float s = 0.f;
    for (int i = threadIdx.x; i < H * dim; i += NT) {
        const float v = ld(row, q_off + i);
        s += v * v;
    }
    const float qinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)(H * dim) + eps);
    s = 0.f;
    for (int i = threadIdx.x; i < G * dim; i += NT) {
        const float v = ld(row, k_off + i);
        s += v * v;
    }
    const float kinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)(G * dim) + eps);
    for (int idx = threadIdx.x; idx < H * R; idx += NT) {
        const int h = idx / R, c = idx - h * R;
        const int e = h * dim + c - vdim;
        qf[t * H * (size_t)R + idx] = c < vdim ? 0.f : ld(row, q_off + e) * qinv * ld(q_w, e) * scale;
    }
    const size_t dst = (size_t)slot[t];
    for (int idx = threadIdx.x; idx < G * R; idx += NT) {
        const int g = idx / R, c = idx - g * R;
        float val;
        if (c < vdim) {
            val = ld(row, v_off + g * vdim + c);
            if (v_first) val = (1.0f - mix) * val + mix * ld(v_first, t * vf_stride + g * vdim + c);
        } else {
            const int e = g * dim + c - vdim;
            val = ld(row, k_off + e) * kinv * ld(k_w, e);
        }
        st(pool, ((size_t)g * pool_rows + dst) * R + c, val);
    }
}
extern "C" int qsv_normed_attention_prep(float* qf, void* pool, int64_t pool_rows, const void* proj, int64_t stride, int q_off,
                                         int k_off, int v_off, int heads, int kv_heads, int dim, int vdim, const void* q_w,
                                         const void* k_w, float eps, float scale, const void* v_first, int64_t vf_stride, float mix,
                                         const int64_t* slot, int n, int dtype, void* stream) {
    QSV_REQUIRE(qf && pool && proj && q_w && k_w && slot, "qsv_normed_attention_prep: null argument");
    QSV_REQUIRE(heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && q_off >= 0 && k_off >= 0 && v_off >= 0 &&
                    q_off + (int64_t)heads * dim <= stride && k_off + (int64_t)kv_heads * dim <= stride &&
                    v_off + (int64_t)kv_heads * vdim <= stride && n >= 0 && (!v_first || vf_stride >= (int64_t)kv_heads * vdim),
                "qsv_normed_attention_prep: bad sizes");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_normed_attention_prep",
                 hipLaunchKernelGGL(normed_attention_prep_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, qf, (T*)pool, pool_rows,
                                    (const T*)proj, stride, q_off, k_off, v_off, heads, kv_heads, dim, vdim, (const T*)q_w,
                                    (const T*)k_w, eps, scale, (const T*)v_first, vf_stride, mix, slot));
    return qsv_launch_status("qsv_normed_attention_prep");
}

// ---- sublayers between two norms: x += rms_norm(y) * w_post; h = rms_norm(x) * w_next ---------------------------------------------
// One workgroup per token, the row in registers (VPT groups of four values per thread; VPT = 0: any width, values re-read).  A
// weight is one gain (wide 0) or one per coordinate.
template <typename T>
__device__ __forceinline__ float4 gain4(const T* w, int wide, int i) {
    if (wide) return ld4v(w, i);
    const float g = ld(w, 0);
    return make_float4(g, g, g, g);
}
template <typename T, int VPT>
__global__ __launch_bounds__(NT) void add_normed_rms_norm_vec_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ y,
                                                                     const T* __restrict__ w_post, int post_wide,
                                                                     const T* __restrict__ w_next, int next_wide, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float4 v[VPT];
    float s = 0.f;
    if (y) {
        float4 u[VPT];
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = (threadIdx.x + k * NT) * 4;
            if (i >= D) continue;
            u[k] = ld4v(y, t * D + i);
            s += u[k].x * u[k].x + u[k].y * u[k].y + u[k].z * u[k].z + u[k].w * u[k].w;
        }
        const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
        s = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = (threadIdx.x + k * NT) * 4;
            if (i >= D) continue;
            const float4 g = gain4(w_post, post_wide, i);
            v[k] = ld4v(x, t * D + i);
            v[k].x += u[k].x * inv * g.x; v[k].y += u[k].y * inv * g.y; v[k].z += u[k].z * inv * g.z; v[k].w += u[k].w * inv * g.w;
            st4v(x, t * D + i, v[k]);
            s += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
        }
    } else {
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = (threadIdx.x + k * NT) * 4;
            if (i >= D) continue;
            v[k] = ld4v(x, t * D + i);
            s += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
        }
    }
    if (!h) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        const float4 g = gain4(w_next, next_wide, i);
        st4v(h, t * D + i, make_float4(v[k].x * inv * g.x, v[k].y * inv * g.y, v[k].z * inv * g.z, v[k].w * inv * g.w));
    }
}
template <typename T>
__global__ __launch_bounds__(NT) void add_normed_rms_norm_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ y,
                                                                 const T* __restrict__ w_post, int post_wide,
                                                                 const T* __restrict__ w_next, int next_wide, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float s = 0.f;
    if (y) {
        for (int i = threadIdx.x; i < D; i += NT) {
            const float u = ld(y, t * D + i);
            s += u * u;
        }
        const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
        s = 0.f;
        for (int i = threadIdx.x; i < D; i += NT) {
            const float v = x[t * D + i] + ld(y, t * D + i) * inv * ld(w_post, post_wide ? i : 0);
            x[t * D + i] = v;
            s += v * v;
        }
    } else {
        for (int i = threadIdx.x; i < D; i += NT) s += x[t * D + i] * x[t * D + i];
    }
    if (!h) return;
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) st(h, t * D + i, x[t * D + i] * inv * ld(w_next, next_wide ? i : 0));
}
extern "C" int qsv_add_normed_rms_norm(float* x, void* h, const void* y, const void* w_post, int post_wide, const void* w_next,
                                       int next_wide, float eps, int n, int D, int dtype, void* stream) {
    QSV_REQUIRE(x && n >= 0 && D > 0 && (!h || w_next) && (!y || w_post), "qsv_add_normed_rms_norm: bad arguments");
    if (n == 0) return QSV_OK;
    const int vecs = (D / 4 + NT - 1) / NT;
    if (D % 4 == 0 && vecs <= 8) {
#define QSV_ANR(V)                                                                                                               \
    QSV_DISPATCH(dtype, "qsv_add_normed_rms_norm",                                                                               \
                 hipLaunchKernelGGL((add_normed_rms_norm_vec_kernel<T, V>), dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, \
                                    (const T*)y, (const T*)w_post, post_wide, (const T*)w_next, next_wide, eps, D))
        if (vecs <= 1) QSV_ANR(1);
        else if (vecs <= 2) QSV_ANR(2);
        else if (vecs <= 4) QSV_ANR(4);
        else QSV_ANR(8);
#undef QSV_ANR
        return qsv_launch_status("qsv_add_normed_rms_norm");
    }
    QSV_DISPATCH(dtype, "qsv_add_normed_rms_norm",
                 hipLaunchKernelGGL(add_normed_rms_norm_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)y,
                                    (const T*)w_post, post_wide, (const T*)w_next, next_wide, eps, D));
    return qsv_launch_status("qsv_add_normed_rms_norm");
}

// ---- query / key norms (per head or over the projection), rotated pairs, cache write -----------------------------------------------
// q_b / k_b / v_b (each may be NULL) are added to the projections first; the pairs are neighbours or, with `halves`, (i, i + rot_n / 2);
// head_scale (may be NULL) multiplies the common scale; a query row starts with q_pad zeros.  One workgroup per token.  Statistics: per head a wave's sum over `dim`; over the projection a workgroup sum.  The rotation works
// (rot_gain > 0, per-head norms only: the norm follows the rotation - its statistic is taken before it, the rotated dimensions weighted by
// rot_gain, the square of the magnitude cos and sin carry, and the turned values are scaled; no weights: q_w, k_w NULL; q_out: the queries
// leave in the storage type)
// on normed values staged in LDS (a pair's two values may sit in different threads).  Dynamic LDS: (heads + kv_heads) * dim floats.
// VEC (every size, stride and address a multiple of four elements, dim <= 256): four elements per lane, dim / 4 lanes (rounded up to a
// power of two, `lph`) per head for the per-head statistics, 16-byte stores.
template <typename T, typename TI, bool VEC>
__global__ __launch_bounds__(NT) void qk_norm_rope_prep_kernel(float* __restrict__ qf, const TI* __restrict__ q, int64_t q_stride,
                                                               const TI* __restrict__ k, int64_t k_stride, const TI* __restrict__ v,
                                                               int64_t v_stride, int H, int G, int dim, int vdim,
                                                               const T* __restrict__ q_w, const T* __restrict__ k_w, int per_head,
                                                               float eps, const float* __restrict__ rope, int rot_n, float scale,
                                                               T* __restrict__ pool, int64_t pool_rows,
                                                               const int64_t* __restrict__ slot, const int32_t* __restrict__ pos,
                                                               const T* __restrict__ q_b, const T* __restrict__ k_b,
                                                               const T* __restrict__ v_b, int halves,
                                                               const float* __restrict__ head_scale, int q_pad, int lph,
                                                               float rot_gain, T* __restrict__ q_out) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
    const int NH = k ? H + G : H;                      // heads staged: the queries', then the keys'
    float* nq = sm;                                    // [NH][dim]
    const TI* qrow = q + t * q_stride;
    const TI* krow = k ? k + t * k_stride : nullptr;
    if (VEC && per_head) {
        const int e = (lane & (lph - 1)) * 4;
        for (int h0 = threadIdx.x / lph; h0 - lane / lph < NH; h0 += NT / lph) {      // (a wave stays together: its lanes exchange sums)
            const bool ok = h0 < NH && e < dim, isq = h0 < H;
            const int hh = isq ? h0 : h0 - H;
            float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
            if (ok) {
                u = ld4v(isq ? qrow : krow, (size_t)hh * dim + e);
                const T* bias = isq ? q_b : k_b;
                if (bias) {
                    const float4 b = ld4v(bias, (size_t)hh * dim + e);
                    u.x += b.x; u.y += b.y; u.z += b.z; u.w += b.w;
                }
            }
            float s;
            if (rot_gain > 0.f)
                s = (e < rot_n ? rot_gain : 1.f) * u.x * u.x + (e + 1 < rot_n ? rot_gain : 1.f) * u.y * u.y +
                    (e + 2 < rot_n ? rot_gain : 1.f) * u.z * u.z + (e + 3 < rot_n ? rot_gain : 1.f) * u.w * u.w;
            else
                s = u.x * u.x + u.y * u.y + u.z * u.z + u.w * u.w;
            for (int o = lph >> 1; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
            const float inv = 1.0f / sqrtf(s / (float)dim + eps);
            if (ok) {
                const float4 g = q_w ? ld4v(isq ? q_w : k_w, e) : make_float4(1.f, 1.f, 1.f, 1.f);
                *(float4*)(nq + h0 * dim + e) = make_float4(u.x * (inv * g.x), u.y * (inv * g.y), u.z * (inv * g.z), u.w * (inv * g.w));
            }
        }
    } else if (per_head) {
        for (int hh = wv; hh < NH; hh += NT / 64) {
            const bool isq = hh < H;
            const TI* src = isq ? qrow + (size_t)hh * dim : krow + (size_t)(hh - H) * dim;
            const T* w = isq ? q_w : k_w;
            const T* bias = isq ? q_b : k_b;
            const int b0 = (isq ? hh : hh - H) * dim;
            float s = 0.f;
            for (int e = lane; e < dim; e += 64) {
                const float u = ld(src, e) + (bias ? ld(bias, b0 + e) : 0.f);
                nq[hh * dim + e] = u;
                s += (rot_gain > 0.f && e < rot_n ? rot_gain : 1.f) * u * u;
            }
            const float inv = 1.0f / sqrtf(wave_sum(s) / (float)dim + eps);
            for (int e = lane; e < dim; e += 64) nq[hh * dim + e] *= q_w ? inv * ld(w, e) : inv;
        }
    } else {
        float s = 0.f;
        for (int i = threadIdx.x; i < H * dim; i += NT) {
            const float u = ld(qrow, i) + (q_b ? ld(q_b, i) : 0.f);
            nq[i] = u;
            s += u * u;
        }
        const float qinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)(H * dim) + eps);
        for (int i = threadIdx.x; i < H * dim; i += NT) nq[i] *= qinv * ld(q_w, i);
        if (k) {
            s = 0.f;
            for (int i = threadIdx.x; i < G * dim; i += NT) {
                const float u = ld(krow, i) + (k_b ? ld(k_b, i) : 0.f);
                nq[H * dim + i] = u;
                s += u * u;
            }
            const float kinv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)(G * dim) + eps);
            for (int i = threadIdx.x; i < G * dim; i += NT) nq[H * dim + i] *= kinv * ld(k_w, i);
        }
    }
    __syncthreads();
    if (rope) {                                        // each pair by one thread
        const int half = rot_n / 2;
        const float* cs = rope + (size_t)pos[t] * rot_n;
        for (int idx = threadIdx.x; idx < NH * half; idx += NT) {
            const int hh = idx / half, i = idx - hh * half;
            const float c = cs[i], sn = cs[half + i];
            const int i0 = hh * dim + (halves ? i : 2 * i), i1 = i0 + (halves ? half : 1);
            const float a = nq[i0], b = nq[i1];
            nq[i0] = a * c - b * sn;
            nq[i1] = b * c + a * sn;
        }
        __syncthreads();
    }
    const int RQ = q_pad + dim, R = vdim + dim;
    if (VEC) {
        const int q4 = RQ >> 2, r4 = R >> 2;
        for (int idx = threadIdx.x; idx < H * q4; idx += NT) {
            const int h = idx / q4, c = (idx - h * q4) * 4;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (c >= q_pad) {
                v = *(const float4*)(nq + h * dim + c - q_pad);
                const float f = head_scale ? scale * head_scale[h] : scale;
                v.x *= f; v.y *= f; v.z *= f; v.w *= f;
            }
            if (q_out) st4v(q_out, t * H * (size_t)RQ + (size_t)idx * 4, v);
            else st4v(qf, t * H * (size_t)RQ + (size_t)idx * 4, v);
        }
        if (!k) return;
        const size_t row = (size_t)slot[t];
        for (int idx = threadIdx.x; idx < G * r4; idx += NT) {
            const int g = idx / r4, c = (idx - g * r4) * 4;
            float4 u;
            if (c < vdim) {
                u = ld4v(v + t * v_stride, (size_t)g * vdim + c);
                if (v_b) {
                    const float4 b = ld4v(v_b, (size_t)g * vdim + c);
                    u.x += b.x; u.y += b.y; u.z += b.z; u.w += b.w;
                }
            } else {
                u = *(const float4*)(nq + (H + g) * dim + c - vdim);
            }
            st4v(pool, ((size_t)g * pool_rows + row) * R + c, u);
        }
        return;
    }
    for (int idx = threadIdx.x; idx < H * RQ; idx += NT) {
        const int h = idx / RQ, c = idx - h * RQ;
        const float qv = c < q_pad ? 0.f : nq[h * dim + c - q_pad] * (head_scale ? scale * head_scale[h] : scale);
        if (q_out) st(q_out, t * H * (size_t)RQ + idx, qv);
        else qf[t * H * (size_t)RQ + idx] = qv;
    }
    if (!k) return;
    const size_t dst = (size_t)slot[t];
    const TI* vrow = v + t * v_stride;
    for (int idx = threadIdx.x; idx < G * R; idx += NT) {
        const int g = idx / R, c = idx - g * R;
        st(pool, ((size_t)g * pool_rows + dst) * R + c,
           c < vdim ? ld(vrow, g * vdim + c) + (v_b ? ld(v_b, g * vdim + c) : 0.f) : nq[(H + g) * dim + c - vdim]);
    }
}
extern "C" int qsv_qk_norm_rope_prep(void* qf, const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v,
                                     int64_t v_stride, int qkv_dtype, int heads, int kv_heads, int dim, int vdim, const void* q_w,
                                     const void* k_w, int per_head, float eps, const float* rope, int rot_n, float scale, void* pool,
                                     int64_t pool_rows, const int64_t* slot, const int32_t* pos, int n, const void* q_b, const void* k_b,
                                     const void* v_b, int halves, const float* head_scale, int q_pad, float rot_gain, int q_store,
                                     int dtype, void* stream) {
    QSV_REQUIRE(qf && q && pos, "qsv_qk_norm_rope_prep: null argument");
    QSV_REQUIRE(!k || (v && pool && slot && !k_w == !q_w), "qsv_qk_norm_rope_prep: keys without values, weight, pool or rows");
    QSV_REQUIRE(q_w || per_head, "qsv_qk_norm_rope_prep: a norm over the projection without its weight");
    QSV_REQUIRE(!(rot_gain > 0.f) || (per_head && !q_w), "qsv_qk_norm_rope_prep: a norm behind the rotation is per head and has no weight");
    if (!rope) rot_n = 0;
    QSV_REQUIRE(heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && n >= 0 && q_pad >= 0 && q_stride >= (int64_t)heads * dim &&
                    (!k || (k_stride >= (int64_t)kv_heads * dim && v_stride >= (int64_t)kv_heads * vdim)),
                "qsv_qk_norm_rope_prep: bad sizes");
    QSV_REQUIRE(!rope || (rot_n > 0 && rot_n % 2 == 0 && rot_n <= dim), "qsv_qk_norm_rope_prep: %d rotated dimensions of %d", rot_n, dim);
    QSV_REQUIRE(qkv_dtype == dtype || qkv_dtype == QSV_F32, "qsv_qk_norm_rope_prep: projections of type %d with storage type %d",
                qkv_dtype, dtype);
    const size_t lds = (size_t)(heads + kv_heads) * dim * 4;
    QSV_REQUIRE(lds <= 64 * 1024, "qsv_qk_norm_rope_prep: %d + %d heads of %d do not fit the workgroup's LDS", heads, kv_heads, dim);
    if (n == 0) return QSV_OK;
    // four elements at a time where everything is aligned to that
    const size_t el = qkv_dtype == QSV_F32 ? 4 : 2, es = dtype == QSV_F32 ? 4 : 2;
    auto al = [](const void* p, size_t size) { return (uintptr_t)p % (4 * size) == 0; };
    const bool vec = dim % 4 == 0 && vdim % 4 == 0 && q_pad % 4 == 0 && dim <= 256 && q_stride % 4 == 0 && al(q, el) && al(q_w, es) && al(q_b, es) &&
                     (!k || (k_stride % 4 == 0 && v_stride % 4 == 0 && al(k, el) && al(v, el) && al(k_w, es) && al(k_b, es) && al(v_b, es) && al(pool, es)));
    int lph = 1;
    while (lph * 4 < dim) lph <<= 1;
#define QSV_QKP(TI, VEC)                                                                                                         \
    QSV_DISPATCH(dtype, "qsv_qk_norm_rope_prep",                                                                                 \
                 hipLaunchKernelGGL((qk_norm_rope_prep_kernel<T, TI, VEC>), dim3(n), dim3(NT), lds, (hipStream_t)stream, q_store ? nullptr : (float*)qf, (const TI*)q, \
                                    q_stride, (const TI*)k, k_stride, (const TI*)v, v_stride, heads, kv_heads, dim, vdim,          \
                                    (const T*)q_w, (const T*)k_w, per_head, eps, rope, rot_n, scale, (T*)pool, pool_rows, slot, pos,  \
                                    (const T*)q_b, (const T*)k_b, (const T*)v_b, halves, head_scale, q_pad, lph, rot_gain,              \
                                    q_store ? (T*)qf : nullptr))
    if (vec) {
        if (qkv_dtype == QSV_F32) QSV_QKP(float, true);
        else QSV_QKP(bf16_t, true);
    } else {
        if (qkv_dtype == QSV_F32) QSV_QKP(float, false);
        else QSV_QKP(bf16_t, false);
    }
#undef QSV_QKP
    return qsv_launch_status("qsv_qk_norm_rope_prep");
}


// ---- embedding with a norm: x = rms_norm(table[token]) * w -------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(NT) void embed_rms_norm_kernel(float* __restrict__ x, const T* __restrict__ table,
                                                            const int32_t* __restrict__ tokens, const T* __restrict__ w, float eps, int D) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    const T* row = table + (size_t)tokens[t] * D;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) s += ld(row, i) * ld(row, i);
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) x[t * D + i] = ld(row, i) * inv * ld(w, i);
}
extern "C" int qsv_embed_rms_norm(float* x, const void* table, const int32_t* tokens, const void* w, float eps, int n, int D, int dtype,
                                  void* stream) {
    QSV_REQUIRE(x && table && tokens && w && n >= 0 && D > 0, "qsv_embed_rms_norm: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_embed_rms_norm",
                 hipLaunchKernelGGL(embed_rms_norm_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (const T*)table, tokens,
                                    (const T*)w, eps, D));
    return qsv_launch_status("qsv_embed_rms_norm");
}

// ---- a token's row plus its causal convolution over time: h_t = x_t + sum_j w[j] x_(t - past + j),  j = 0 .. past = taps - 1 ------------
// Inputs before a run's start come from the sequence's history (rows of `past` inputs, oldest first; none at the sequence's start);
// a run's last token writes the new history into the state's other copy.
struct ConvState {
    const float* w;                 // [taps, D]
    float* hist;                    // [2 slots, past, D]
    const int32_t *run_off, *rd, *wr;
    int past;
};
// the input d tokens before token t (the i-th of its run), channels c .. c + 3 (V4) or c
__device__ __forceinline__ float4 conv_in4(const float* x, const ConvState& cv, size_t t, int i, int rd, int d, int D, int c) {
    if (d <= i) return ld4v(x, (t - d) * (size_t)D + c);
    if (rd >= 0) return ld4v(cv.hist, ((size_t)rd * cv.past + (cv.past + i - d)) * D + c);
    return make_float4(0.f, 0.f, 0.f, 0.f);
}
__device__ __forceinline__ float conv_in1(const float* x, const ConvState& cv, size_t t, int i, int rd, int d, int D, int c) {
    if (d <= i) return x[(t - d) * (size_t)D + c];
    return rd >= 0 ? cv.hist[((size_t)rd * cv.past + (cv.past + i - d)) * D + c] : 0.f;
}
// h of channels c .. c + 3 of token t, whose own row holds v there; writes the history if the token ends its run
template <typename T>
__device__ __forceinline__ void conv_tail4(T* h, const float* x, const ConvState& cv, size_t t, int i, int rd, int wr, int D, int c, float4 v) {
    const float4 w0 = ld4v(cv.w, (size_t)cv.past * D + c);
    float4 a = make_float4(v.x + w0.x * v.x, v.y + w0.y * v.y, v.z + w0.z * v.z, v.w + w0.w * v.w);
    for (int d = 1; d <= cv.past; ++d) {
        const float4 u = conv_in4(x, cv, t, i, rd, d, D, c), w = ld4v(cv.w, (size_t)(cv.past - d) * D + c);
        a.x += w.x * u.x; a.y += w.y * u.y; a.z += w.z * u.z; a.w += w.w * u.w;
        if (wr >= 0 && d < cv.past) st4v(cv.hist, ((size_t)wr * cv.past + (cv.past - 1 - d)) * D + c, u);
    }
    if (wr >= 0 && cv.past > 0) st4v(cv.hist, ((size_t)wr * cv.past + cv.past - 1) * D + c, v);
    st4v(h, t * D + c, a);
}
template <typename T>
__device__ __forceinline__ void conv_tail1(T* h, const float* x, const ConvState& cv, size_t t, int i, int rd, int wr, int D, int c, float v) {
    float a = v + cv.w[(size_t)cv.past * D + c] * v;
    for (int d = 1; d <= cv.past; ++d) {
        const float u = conv_in1(x, cv, t, i, rd, d, D, c);
        a += cv.w[(size_t)(cv.past - d) * D + c] * u;
        if (wr >= 0 && d < cv.past) cv.hist[((size_t)wr * cv.past + (cv.past - 1 - d)) * D + c] = u;
    }
    if (wr >= 0 && cv.past > 0) cv.hist[((size_t)wr * cv.past + cv.past - 1) * D + c] = v;
    st(h, t * D + c, a);
}
template <typename T, bool VEC>
__global__ __launch_bounds__(NT) void residual_conv_kernel(T* __restrict__ h, const float* __restrict__ x, ConvState cv, int D) {
    const size_t t = blockIdx.x;
    const int i = cv.run_off[t], rd = cv.rd[t], wr = cv.wr[t];
    if (VEC) {
        for (int c = threadIdx.x * 4; c < D; c += NT * 4) conv_tail4(h, x, cv, t, i, rd, wr, D, c, ld4v(x, t * D + c));
    } else {
        for (int c = threadIdx.x; c < D; c += NT) conv_tail1(h, x, cv, t, i, rd, wr, D, c, x[t * D + c]);
    }
}
// The same for PAST = taps - 1 known and widths of multiples of four: a workgroup walks CONV_TB consecutive tokens of four channels per
// thread, the last PAST rows in registers - every row is read once (and PAST more at a block's start); all CONV_TB rows are requested
// at once.  Rows of another run in the registers are replaced by the run's history (or zeros).
constexpr int CONV_TB = 8;
template <typename T, int PAST>
__global__ __launch_bounds__(NT) void residual_conv_rows_kernel(T* __restrict__ h, const float* __restrict__ x, ConvState cv, int n, int D) {
    const int c = ((int)blockIdx.y * NT + (int)threadIdx.x) * 4;
    if (c >= D) return;
    const int t0 = (int)blockIdx.x * CONV_TB, cnt = min(CONV_TB, n - t0);
    float4 w[PAST + 1], r[CONV_TB + PAST];               // r[PAST + k]: row t0 + k
#pragma unroll
    for (int j = 0; j <= PAST; ++j) w[j] = ld4v(cv.w, (size_t)j * D + c);
#pragma unroll
    for (int k = 0; k < CONV_TB + PAST; ++k) r[k] = ld4v(x, (size_t)min(max(t0 - PAST + k, 0), n - 1) * D + c);
#pragma unroll
    for (int k = 0; k < CONV_TB; ++k) {
        if (k >= cnt) continue;
        const size_t t = (size_t)(t0 + k);
        const int i = cv.run_off[t], wr = cv.wr[t];      // (uniform over the workgroup)
        float4 u[PAST + 1];                              // u[d]: the input d tokens back
#pragma unroll
        for (int d = 0; d <= PAST; ++d) u[d] = r[PAST + k - d];
        if (i < PAST) {
            const int rd = cv.rd[t];
#pragma unroll
            for (int d = 1; d <= PAST; ++d)
                if (d > i) u[d] = conv_in4(x, cv, t, i, rd, d, D, c);
        }
        float4 a = u[0];
#pragma unroll
        for (int d = 0; d <= PAST; ++d) {
            const float4 wd = w[PAST - d];
            a.x += wd.x * u[d].x; a.y += wd.y * u[d].y; a.z += wd.z * u[d].z; a.w += wd.w * u[d].w;
        }
        st4v(h, t * D + c, a);
        if (wr >= 0) {
#pragma unroll
            for (int d = 0; d < PAST; ++d) st4v(cv.hist, ((size_t)wr * PAST + (PAST - 1 - d)) * D + c, u[d]);
        }
    }
}
extern "C" int qsv_residual_conv(void* h, const float* x, const float* w, int taps, float* hist, const int32_t* run_off,
                                 const int32_t* state_rd, const int32_t* state_wr, int n, int D, int dtype, void* stream) {
    QSV_REQUIRE(h && x && w && run_off && state_rd && state_wr && n >= 0 && D > 0 && taps >= 1 && (taps == 1 || hist),
                "qsv_residual_conv: bad arguments");
    if (n == 0) return QSV_OK;
    const ConvState cv = {w, hist, run_off, state_rd, state_wr, taps - 1};
    if (D % 4 == 0 && taps >= 2 && taps <= 4 && n >= 2 * CONV_TB && D <= 65535 * NT * 4) {
        const dim3 grid((n + CONV_TB - 1) / CONV_TB, (D / 4 + NT - 1) / NT);
#define QSV_RCR(P)                                                                                                          \
    QSV_DISPATCH(dtype, "qsv_residual_conv",                                                                                \
                 hipLaunchKernelGGL((residual_conv_rows_kernel<T, P>), grid, dim3(NT), 0, (hipStream_t)stream, (T*)h, x, cv, n, D))
        if (taps == 2) QSV_RCR(1);
        else if (taps == 3) QSV_RCR(2);
        else QSV_RCR(3);
#undef QSV_RCR
        return qsv_launch_status("qsv_residual_conv");
    }
    if (D % 4 == 0)
        QSV_DISPATCH(dtype, "qsv_residual_conv",
                     hipLaunchKernelGGL((residual_conv_kernel<T, true>), dim3(n), dim3(NT), 0, (hipStream_t)stream, (T*)h, x, cv, D));
    else
        QSV_DISPATCH(dtype, "qsv_residual_conv",
                     hipLaunchKernelGGL((residual_conv_kernel<T, false>), dim3(n), dim3(NT), 0, (hipStream_t)stream, (T*)h, x, cv, D));
    return qsv_launch_status("qsv_residual_conv");
}

// ---- norm after the sum: x = rms_norm(alpha x + y) * w, h = x in the storage type ------------------------------------------------------
// With `cv.w` (steps in which every run is one token: no row of this launch reads another's new x) h is instead the next mixer's
// input, x plus its convolution over time.  The row in registers (VPT groups of four values per thread), or any width.
template <typename T, int VPT>
__global__ __launch_bounds__(NT) void scaled_add_rms_norm_vec_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ y,
                                                                     float alpha, const T* __restrict__ w, float eps, int D, ConvState cv) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float4 v[VPT];
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        const float4 a = ld4v(x, t * D + i), b = ld4v(y, t * D + i);
        v[k] = make_float4(alpha * a.x + b.x, alpha * a.y + b.y, alpha * a.z + b.z, alpha * a.w + b.w);
        s += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
    }
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * NT) * 4;
        if (i >= D) continue;
        const float4 g = ld4v(w, i);
        v[k] = make_float4(v[k].x * inv * g.x, v[k].y * inv * g.y, v[k].z * inv * g.z, v[k].w * inv * g.w);
        st4v(x, t * D + i, v[k]);
        if (!h) continue;
        if (cv.w) conv_tail4(h, x, cv, t, 0, cv.rd[t], cv.wr[t], D, i, v[k]);
        else st4v(h, t * D + i, v[k]);
    }
}
template <typename T>
__global__ __launch_bounds__(NT) void scaled_add_rms_norm_kernel(float* __restrict__ x, T* __restrict__ h, const T* __restrict__ y,
                                                                 float alpha, const T* __restrict__ w, float eps, int D, ConvState cv) {
    __shared__ float red[NT / 64 + 1];
    const size_t t = blockIdx.x;
    float s = 0.f;
    for (int i = threadIdx.x; i < D; i += NT) {
        const float v = alpha * x[t * D + i] + ld(y, t * D + i);
        s += v * v;
    }
    const float inv = 1.0f / sqrtf(block_sum<NT>(s, red) / (float)D + eps);
    for (int i = threadIdx.x; i < D; i += NT) {
        const float v = (alpha * x[t * D + i] + ld(y, t * D + i)) * inv * ld(w, i);
        x[t * D + i] = v;
        if (!h) continue;
        if (cv.w) conv_tail1(h, x, cv, t, 0, cv.rd[t], cv.wr[t], D, i, v);
        else st(h, t * D + i, v);
    }
}
extern "C" int qsv_scaled_add_rms_norm(float* x, void* h, const void* y, float alpha, const void* w, float eps, const float* conv_w,
                                       int taps, float* hist, const int32_t* state_rd, const int32_t* state_wr, int n, int D, int dtype,
                                       void* stream) {
    QSV_REQUIRE(x && y && w && n >= 0 && D > 0, "qsv_scaled_add_rms_norm: bad arguments");
    QSV_REQUIRE(!conv_w || (h && taps >= 1 && state_rd && state_wr && (taps == 1 || hist)),
                "qsv_scaled_add_rms_norm: a convolution without its state or output");
    if (n == 0) return QSV_OK;
    const ConvState cv = {conv_w, hist, nullptr, state_rd, state_wr, conv_w ? taps - 1 : 0};
    const int vecs = (D / 4 + NT - 1) / NT;
    if (D % 4 == 0 && vecs <= 8) {
#define QSV_SAN(V)                                                                                                               \
    QSV_DISPATCH(dtype, "qsv_scaled_add_rms_norm",                                                                               \
                 hipLaunchKernelGGL((scaled_add_rms_norm_vec_kernel<T, V>), dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, \
                                    (const T*)y, alpha, (const T*)w, eps, D, cv))
        if (vecs <= 1) QSV_SAN(1);
        else if (vecs <= 2) QSV_SAN(2);
        else if (vecs <= 4) QSV_SAN(4);
        else QSV_SAN(8);
#undef QSV_SAN
        return qsv_launch_status("qsv_scaled_add_rms_norm");
    }
    QSV_DISPATCH(dtype, "qsv_scaled_add_rms_norm",
                 hipLaunchKernelGGL(scaled_add_rms_norm_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, x, (T*)h, (const T*)y,
                                    alpha, (const T*)w, eps, D, cv));
    return qsv_launch_status("qsv_scaled_add_rms_norm");
}

// ---- retention operands: queries and keys turned by the position (halves layout), everything float --------------------------------------
// out[t] = [ rot(q[t]) (H dim) | rot(k[t]) (H dim) | v[t] (H vdim) ]; rope float [positions, 2, rot_n / 2] or NULL.
template <typename T>
__global__ __launch_bounds__(NT) void rotate_qk_kernel(float* __restrict__ out, const T* __restrict__ qkv, int64_t stride, int heads2,
                                                       int dim, int n_v, const float* __restrict__ rope, int rot_n,
                                                       const int32_t* __restrict__ pos) {
    const size_t t = blockIdx.x;
    const T* row = qkv + t * stride;
    const int nqk = heads2 * dim, half = rot_n >> 1;
    float* o = out + t * (size_t)(nqk + n_v);
    const float* cs = rope ? rope + (size_t)pos[t] * rot_n : nullptr;
    for (int idx = threadIdx.x; idx < heads2 * half; idx += NT) {
        const int hh = idx / half, i = idx - hh * half;
        const float a = ld(row, hh * dim + i), b = ld(row, hh * dim + half + i), c = cs[i], s = cs[half + i];
        o[hh * dim + i] = a * c - b * s;
        o[hh * dim + half + i] = b * c + a * s;
    }
    if (rot_n < dim) {
        const int rest = dim - rot_n;
        for (int idx = threadIdx.x; idx < heads2 * rest; idx += NT) {
            const int hh = idx / rest, i = hh * dim + rot_n + (idx - hh * rest);
            o[i] = ld(row, i);
        }
    }
    for (int i = threadIdx.x; i < n_v; i += NT) o[nqk + i] = ld(row, nqk + i);
}
extern "C" int qsv_rotate_qk(float* out, const void* qkv, int64_t stride, int heads, int dim, int vdim, const float* rope, int rot_n,
                             const int32_t* pos, int n, int dtype, void* stream) {
    QSV_REQUIRE(out && qkv && pos && n >= 0 && heads > 0 && dim > 0 && vdim > 0 && rot_n >= 0 && rot_n % 2 == 0 && rot_n <= dim &&
                    (rope || rot_n == 0) && stride >= (int64_t)heads * (2 * dim + vdim),
                "qsv_rotate_qk: bad arguments");
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_rotate_qk",
                 hipLaunchKernelGGL(rotate_qk_kernel<T>, dim3(n), dim3(NT), 0, (hipStream_t)stream, out, (const T*)qkv, stride, 2 * heads,
                                    dim, heads * vdim, rope, rot_n, pos));
    return qsv_launch_status("qsv_rotate_qk");
}
