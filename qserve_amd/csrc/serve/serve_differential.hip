// serve_differential.hip -- attention whose keys come in one or two maps over the same values, on a paged cache of rows
// [v (vdim) | k_0 (dim) | .. | k_(M-1) (dim)] per key / value head; and the launch that feeds it: a short causal convolution over time on
// every channel of q, k and v, the query's scale and temperature, the cache write.
//
// With two maps ("differential"): a_m = softmax_j(q_m . k_m) v per head, o = a_1 - lambda a_2, o / rms(o) * out_scale * sigmoid(gate).  Both
// maps read the same rows in one pass; the combination, the norm and the gate are the epilogue.  With one map: plain causal attention.
// Scores, maxima, sums, the outputs and their combination are float.
#include "serve_common.h"

#include <type_traits>
#include <utility>

namespace {
constexpr int NT = 256;
constexpr int NW = NT / 64;
constexpr float LOG2E = 1.4426950408889634f;

// ---- convolution over time, scale and temperature, cache write -----------------------------------------------------------------------
// Columns of a projection row: q (Cq channels) | k (G * Dk) | v (G * vdim); y_t = sum_j w[c, j] u_(t - past + j), past = taps - 1.  Inputs before
// a run's start come from the sequence's history ([slots 2, past, C], the projected rows, oldest first; none at the sequence's start); a run's
// last token writes the new history into the state's other copy.  q leaves as the storage type, times scale times (with temp_every > 0)
// 1 + temp_coef ln(floor((p + 1) / temp_every) + 1); k and v go into the cache row of the token.
struct ConvHeads {
    const float* w;                 // [taps, C]
    float* hist;
    const int32_t *run_off, *rd, *wr, *pos;
    const int64_t* slot;
    int64_t stride, pool_rows;
    int past, C, Cq, Dk, vdim, n_kv;      // n_kv: G * Dk (0: queries only)
    float scale, temp_coef;
    double temp_every;
};
__device__ __forceinline__ float query_factor(const ConvHeads& a, int p) {
    if (!(a.temp_every > 0.0)) return a.scale;
    return a.scale * (1.0f + a.temp_coef * logf((float)floor((double)(p + 1) / a.temp_every) + 1.0f));
}
// V consecutive channels
template <int V>
struct Vec {
    float v[V];
};
template <int V>
__device__ __forceinline__ Vec<V> ldv(const float* p, size_t i) {
    Vec<V> r;
    if constexpr (V == 4) {
        const float4 u = *(const float4*)(p + i);
        r = {{u.x, u.y, u.z, u.w}};
    } else {
        for (int e = 0; e < V; ++e) r.v[e] = p[i + e];
    }
    return r;
}
template <int V>
__device__ __forceinline__ Vec<V> ldv(const bf16_t* p, size_t i) {
    Vec<V> r;
    if constexpr (V == 4) {
        const uint2 u = *(const uint2*)(p + i);
        r = {{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u)}};
    } else {
        for (int e = 0; e < V; ++e) r.v[e] = bf2f(p[i + e]);
    }
    return r;
}
template <int V>
__device__ __forceinline__ void stv(float* p, size_t i, const Vec<V>& x) {
    if constexpr (V == 4) *(float4*)(p + i) = make_float4(x.v[0], x.v[1], x.v[2], x.v[3]);
    else
        for (int e = 0; e < V; ++e) p[i + e] = x.v[e];
}
template <int V>
__device__ __forceinline__ void stv(bf16_t* p, size_t i, const Vec<V>& x) {
    if constexpr (V == 4) {
        uint2 u;
        u.x = (uint32_t)f2bf(x.v[0]) | ((uint32_t)f2bf(x.v[1]) << 16);
        u.y = (uint32_t)f2bf(x.v[2]) | ((uint32_t)f2bf(x.v[3]) << 16);
        *(uint2*)(p + i) = u;
    } else {
        for (int e = 0; e < V; ++e) p[i + e] = f2bf(x.v[e]);
    }
}
// the input d tokens before token t (the i-th of its run)
template <int V, typename T>
__device__ __forceinline__ Vec<V> conv_input(const T* proj, const ConvHeads& a, size_t t, int i, int rd, int d, int c) {
    if (d <= i) return ldv<V>(proj, (t - d) * (size_t)a.stride + c);
    if (rd >= 0) return ldv<V>(a.hist, ((size_t)rd * a.past + (a.past + i - d)) * a.C + c);
    Vec<V> z;
#pragma unroll
    for (int e = 0; e < V; ++e) z.v[e] = 0.f;
    return z;
}
template <int V, typename T>
__device__ __forceinline__ void conv_store(T* q, T* pool, const ConvHeads& a, size_t t, int c, Vec<V> y, float qf) {
    if (c < a.Cq) {
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] *= qf;
        stv<V>(q, t * a.Cq + c, y);
        return;
    }
    const int kc = c - a.Cq, R = a.vdim + a.Dk;
    const bool key = kc < a.n_kv;
    const int g = key ? kc / a.Dk : (kc - a.n_kv) / a.vdim;
    const int e0 = key ? a.vdim + kc - g * a.Dk : kc - a.n_kv - g * a.vdim;
    stv<V>(pool, ((size_t)g * a.pool_rows + (size_t)a.slot[t]) * R + e0, y);
}
// workgroup = (token, 256 V channels), any number of taps
template <typename T, int V>
__global__ __launch_bounds__(NT) void conv_heads_kernel(T* __restrict__ q, T* __restrict__ pool, const T* __restrict__ proj, ConvHeads a) {
    const size_t t = blockIdx.x;
    const int c = ((int)blockIdx.y * NT + (int)threadIdx.x) * V;
    if (c >= a.C) return;
    const int i = a.run_off[t], rd = a.rd[t], wr = a.wr[t];
    Vec<V> y, u = ldv<V>(proj, t * (size_t)a.stride + c), w = ldv<V>(a.w, (size_t)a.past * a.C + c);
#pragma unroll
    for (int e = 0; e < V; ++e) y.v[e] = w.v[e] * u.v[e];
    if (wr >= 0 && a.past > 0) stv<V>(a.hist, ((size_t)wr * a.past + a.past - 1) * a.C + c, u);
    for (int d = 1; d <= a.past; ++d) {
        u = conv_input<V>(proj, a, t, i, rd, d, c);
        w = ldv<V>(a.w, (size_t)(a.past - d) * a.C + c);
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += w.v[e] * u.v[e];
        if (wr >= 0 && d < a.past) stv<V>(a.hist, ((size_t)wr * a.past + (a.past - 1 - d)) * a.C + c, u);
    }
    conv_store<V>(q, pool, a, t, c, y, query_factor(a, a.pos[t]));
}
// The same for PAST = taps - 1 known: a workgroup walks TB consecutive tokens of four channels per thread with the last PAST rows in
// registers; rows of another run are replaced by the run's history (or zeros).
constexpr int TB = 8;
template <typename T, int PAST>
__global__ __launch_bounds__(NT) void conv_heads_rows_kernel(T* __restrict__ q, T* __restrict__ pool, const T* __restrict__ proj, ConvHeads a, int n) {
    const int c = ((int)blockIdx.y * NT + (int)threadIdx.x) * 4;
    if (c >= a.C) return;
    const int t0 = (int)blockIdx.x * TB, cnt = min(TB, n - t0);
    Vec<4> w[PAST + 1], r[TB + PAST];                    // r[PAST + k]: row t0 + k
#pragma unroll
    for (int j = 0; j <= PAST; ++j) w[j] = ldv<4>(a.w, (size_t)j * a.C + c);
#pragma unroll
    for (int k = 0; k < TB + PAST; ++k) r[k] = ldv<4>(proj, (size_t)min(max(t0 - PAST + k, 0), n - 1) * (size_t)a.stride + c);
#pragma unroll
    for (int k = 0; k < TB; ++k) {
        if (k >= cnt) continue;
        const size_t t = (size_t)(t0 + k);
        const int i = a.run_off[t], wr = a.wr[t];        // (uniform over the workgroup)
        Vec<4> u[PAST + 1];                              // u[d]: the input d tokens back
#pragma unroll
        for (int d = 0; d <= PAST; ++d) u[d] = r[PAST + k - d];
        if (i < PAST) {
            const int rd = a.rd[t];
#pragma unroll
            for (int d = 1; d <= PAST; ++d)
                if (d > i) u[d] = conv_input<4>(proj, a, t, i, rd, d, c);
        }
        Vec<4> y;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            float s = 0.f;
#pragma unroll
            for (int d = 0; d <= PAST; ++d) s += w[PAST - d].v[e] * u[d].v[e];
            y.v[e] = s;
        }
        if (wr >= 0) {
#pragma unroll
            for (int d = 0; d < PAST; ++d) stv<4>(a.hist, ((size_t)wr * PAST + (PAST - 1 - d)) * a.C + c, u[d]);
        }
        conv_store<4>(q, pool, a, t, c, y, query_factor(a, a.pos[t]));
    }
}

// ---- differential attention, any sizes, both storage types -------------------------------------------------------------------------------
// Workgroup = (token, head), four waves; wave w takes keys KG (w + 4 n) .., lanes spread over a row's elements, one butterfly reduction per
// score, online softmax per map and group of keys, the four partial results merged through LDS.
constexpr int KG = 4;
template <typename T, int EK, int EV>
__global__ __launch_bounds__(NT) void diff_attention_wave_kernel(T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ pool,
                                                                 const int32_t* __restrict__ block_table, int table_stride,
                                                                 const int32_t* __restrict__ seq, const int32_t* __restrict__ pos, int H, int per,
                                                                 int dim, int vdim, int page, int64_t pool_stride, float lambda, float out_scale,
                                                                 float eps, const T* __restrict__ gate, int64_t gate_stride) {
    __shared__ float s_m[2][NW], s_l[2][NW], red[NW + 1];
    __shared__ float s_acc[2][NW][64 * EV];
    const size_t t = blockIdx.x / H;
    const int h = blockIdx.x % H, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int R = vdim + 2 * dim, p = pos[t];
    pool += (size_t)(h / per) * (size_t)pool_stride;
    const int32_t* bt = block_table + (size_t)seq[t] * table_stride;
    float qr[2][EK], acc[2][EV], m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
    for (int f = 0; f < 2; ++f) {
#pragma unroll
        for (int i = 0; i < EK; ++i) {
            const int e = lane + 64 * i;
            qr[f][i] = e < dim ? ld(q, ((t * H + h) * 2 + f) * (size_t)dim + e) : 0.f;
        }
#pragma unroll
        for (int i = 0; i < EV; ++i) acc[f][i] = 0.f;
    }
    for (int j0 = w * KG; j0 <= p; j0 += NW * KG) {
        float v[KG][EV], s[2][KG];
#pragma unroll
        for (int k = 0; k < KG; ++k) {
            const int j = min(j0 + k, p);
            const T* row = pool + ((size_t)bt[j / page] * page + (size_t)(j % page)) * (size_t)R;
#pragma unroll
            for (int i = 0; i < EV; ++i) v[k][i] = lane + 64 * i < vdim ? ld(row, lane + 64 * i) : 0.f;
#pragma unroll
            for (int f = 0; f < 2; ++f) {
                float d = 0.f;
#pragma unroll
                for (int i = 0; i < EK; ++i)
                    if (lane + 64 * i < dim) d += qr[f][i] * ld(row, vdim + f * dim + lane + 64 * i);
                d = wave_sum(d);
                s[f][k] = j0 + k <= p ? d : -INFINITY;
            }
        }
#pragma unroll
        for (int f = 0; f < 2; ++f) {
            float mx = m[f];
#pragma unroll
            for (int k = 0; k < KG; ++k) mx = fmaxf(mx, s[f][k]);
            const float alpha = expf(m[f] - mx);       // first group: exp(-inf) = 0 (mx is finite: key j0 is visible)
            float pk[KG], ps = 0.f;
#pragma unroll
            for (int k = 0; k < KG; ++k) {
                pk[k] = expf(s[f][k] - mx);
                ps += pk[k];
            }
            l[f] = l[f] * alpha + ps;
            m[f] = mx;
#pragma unroll
            for (int i = 0; i < EV; ++i) {
                float a = acc[f][i] * alpha;
#pragma unroll
                for (int k = 0; k < KG; ++k) a += pk[k] * v[k][i];
                acc[f][i] = a;
            }
        }
    }
#pragma unroll
    for (int f = 0; f < 2; ++f) {
        if (lane == 0) {
            s_m[f][w] = m[f];
            s_l[f][w] = l[f];
        }
#pragma unroll
        for (int i = 0; i < EV; ++i) s_acc[f][w][lane + 64 * i] = acc[f][i];
    }
    __syncthreads();
    float fac[2][NW];
#pragma unroll
    for (int f = 0; f < 2; ++f) {
        float M = s_m[f][0], L = 0.f;
#pragma unroll
        for (int k = 1; k < NW; ++k) M = fmaxf(M, s_m[f][k]);
#pragma unroll
        for (int k = 0; k < NW; ++k) {
            fac[f][k] = expf(s_m[f][k] - M);           // a wave without keys has m = -inf: factor 0
            L += fac[f][k] * s_l[f][k];
        }
#pragma unroll
        for (int k = 0; k < NW; ++k) fac[f][k] /= L;
    }
    constexpr int EO = (64 * EV + NT - 1) / NT;
    float o[EO], sq = 0.f;
#pragma unroll
    for (int i = 0; i < EO; ++i) {
        const int e = threadIdx.x + NT * i;
        o[i] = 0.f;
        if (e < vdim) {
            float a1 = 0.f, a2 = 0.f;
#pragma unroll
            for (int k = 0; k < NW; ++k) {
                a1 += fac[0][k] * s_acc[0][k][e];
                a2 += fac[1][k] * s_acc[1][k][e];
            }
            o[i] = a1 - lambda * a2;
        }
        sq += o[i] * o[i];
    }
    const float inv = out_scale / sqrtf(block_sum<NT>(sq, red) / (float)vdim + eps);
#pragma unroll
    for (int i = 0; i < EO; ++i) {
        const int e = threadIdx.x + NT * i;
        if (e >= vdim) continue;
        float y = o[i] * inv;
        if (gate) y /= 1.0f + expf(-ld(gate, t * (size_t)gate_stride + (size_t)h * vdim + e));
        st(out, (t * H + h) * (size_t)vdim + e, y);
    }
}
// ---- matrix-core kernels (bfloat16): M key maps over the same values, dim = 16 DT, vdim = 32 CT ------------------------------------------
// A wave owns 32 query rows = TQ tokens x HP head slots (one pool's heads, rounded up to a power of two; more than 32: head groups) and ALL
// M maps of them, so that a value fragment read from LDS serves M products.  Keys come in blocks of 32 cache rows (the prompt kernel: 64, inside one page), copied
// straight into LDS (global_load_lds) as they lie in memory, 16-byte pieces of a row permuted by the row's number so that neither the
// key reads (16 bytes per lane, 32 rows) nor the transposing value reads (ds_read_b64_tr_b16, 4 rows) pile up on a bank.  S^T = K Q^T
// (v_mfma_f32_32x32x16_bf16) leaves a lane 16 of the 32 scores of its own row; the softmax needs one exchange (lanes ^ 32), the weights
// are the B operand of O^T += V^T P^T as they stand.  The reference maximum moves only when a block exceeds it by more than 2^8.
// * prompt kernel: a workgroup's four waves own four groups of rows of one sequence and share two-block tiles, double-buffered, one barrier a
//   tile; the epilogue combines the maps in registers.  Workgroups are numbered so that a sequence's tiles share an XCD's L2.
// * step kernel (runs of at most TQ tokens: decoding): the four waves own the SAME rows and walk different key blocks, each through buffers of
//   its own without any barrier, and merge at the end; key splits over workgroups leave partial results for a merge launch.
typedef float v16f __attribute__((ext_vector_type(16)));
typedef float f2v __attribute__((ext_vector_type(2)));
typedef __bf16 b2v __attribute__((ext_vector_type(2)));
typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef unsigned int v4u __attribute__((ext_vector_type(4)));
typedef unsigned int v2u __attribute__((ext_vector_type(2)));
typedef short s4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s4* lds_s4;
typedef __attribute__((address_space(3))) void* lds_ptr;

constexpr int BN = 32;                                   // keys per block
__device__ __forceinline__ unsigned pack_bf2(float a, float b) { return __builtin_bit_cast(unsigned, __builtin_convertvector((f2v{a, b}), b2v)); }

template <int DT, int CT, int M>
struct Shape {
    static constexpr int DIM = 16 * DT, VDIM = 32 * CT;
    static constexpr int PPR = 4 * CT + 2 * M * DT;      // 16-byte pieces of a row
    static constexpr int BLOCK = BN * PPR * 16;          // bytes of a block
    static constexpr int XM = (PPR % 16 == 0 ? 16 : PPR % 8 == 0 ? 8 : PPR % 4 == 0 ? 4 : 2) - 1;
    __device__ static __forceinline__ int swizzle(int row) { return (((row & 3) << 2) | ((row >> 2) & 3)) & XM; }
    static constexpr int BUFS = 8 * BLOCK <= 144 * 1024 ? 2 : 1;                     // step kernel: buffers per wave
    static constexpr int OROW = VDIM + 4;                // merge: floats per row
    static constexpr int MERGE = NW * M * 32 * OROW * 4, ML = NW * M * 32 * 2 * 4;   // bytes
    static constexpr int STEP_LDS = (NW * BUFS * BLOCK > MERGE ? NW * BUFS * BLOCK : MERGE) + ML;
    static constexpr int PROMPT_LDS = 4 * BLOCK;
    static constexpr int REGS = 16 * M * CT + 4 * M * DT;                            // accumulators + query fragments
    static constexpr int PROMPT_OCC = PROMPT_LDS <= 80 * 1024 && REGS <= 168 ? 2 : 1;
    static constexpr int STEP_OCC = STEP_LDS <= 80 * 1024 && REGS <= 168 ? 2 : 1;
};

struct MapsArgs {
    bf16_t* out;
    const bf16_t *q, *pool, *gate;
    const int32_t *block_table, *pos, *tiles;
    float *part_o, *part_ml;
    int64_t pool_stride, gate_stride;
    int table_stride, n_tiles, H, per, page_shift, HP, TQ, HG, Z;
    float lambda, out_scale, eps;
};

// x ^ N, kept out of the compiler's sight: it would hold every such address of the key loop in a register of its own and spill accumulators
template <int N>
__device__ __forceinline__ unsigned flip(unsigned x) {
    if constexpr (N != 0) asm volatile("v_xor_b32 %0, %1, %0" : "+v"(x) : "n"(N));
    return x;
}
template <int N, class F, int... I>
__device__ __forceinline__ void each_of(F&& f, std::integer_sequence<int, I...>) {
    (f(std::integral_constant<int, I>{}), ...);
}
template <int N, class F>
__device__ __forceinline__ void each(F&& f) {            // f(0), .., f(N - 1) with compile-time arguments
    each_of<N>(f, std::make_integer_sequence<int, N>{});
}

template <int DT, int CT, int M>
struct Rows {                                            // the softmax state of a wave's 32 rows
    using S = Shape<DT, CT, M>;
    v4u qf[M][DT];
    v16f o[M][CT];
    float m[M], l[M];

    __device__ __forceinline__ void start(const bf16_t* qrow, bool ok, int hi) {
#pragma unroll
        for (int f = 0; f < M; ++f) {
#pragma unroll
            for (int s = 0; s < DT; ++s) qf[f][s] = ok ? *(const v4u*)(qrow + f * S::DIM + 16 * s + 8 * hi) : v4u{0u, 0u, 0u, 0u};
#pragma unroll
            for (int c = 0; c < CT; ++c)
#pragma unroll
                for (int r = 0; r < 16; ++r) o[f][c][r] = 0.f;
            m[f] = -INFINITY;
            l[f] = 0.f;
        }
    }
    // keys k0 .. k0 + 31, staged at `blk`; p_row: this lane's position; mask: some row of the wave does not see the whole block
    __device__ __forceinline__ void block(const unsigned char* blk, int k0, int p_row, bool mask, int lane) {
        const int li = lane & 31, hi = lane >> 5;
        const unsigned char* krow = blk + li * (S::PPR * 16);
        const unsigned kcol = (unsigned)((hi ^ S::swizzle(li)) * 16);
        unsigned pb[M][2][4];
        each<M>([&](auto fc) {
            constexpr int f = decltype(fc)::value;
            v16f sc;
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[r] = 0.f;
            each<DT>([&](auto st) {                                      // (piece 4 CT + 2 DT f + 2 s + hi of the row: an even number plus hi)
                constexpr int s = decltype(st)::value;
                const v4u a = *(const v4u*)(krow + flip<(4 * CT + 2 * DT * f + 2 * s) * 16>(kcol));
                sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf8, a), __builtin_bit_cast(bf8, qf[f][s]), sc, 0, 0, 0);
            });
            // sc[r]: key k0 + (r & 3) + 8 (r >> 2) + 4 hi of this lane's row
            float mx = -INFINITY;
            if (mask) {
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    sc[r] = k0 + (r & 3) + 8 * (r >> 2) + 4 * hi <= p_row ? sc[r] : -INFINITY;
                    mx = fmaxf(mx, sc[r]);
                }
            } else {
#pragma unroll
                for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sc[r]);
            }
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64)) * LOG2E;
            const float mn = mx > m[f] + 8.0f ? mx : m[f];
            const float mu = mn == -INFINITY ? 0.f : mn;                 // (nothing seen so far)
            const float alpha = __builtin_amdgcn_exp2f(m[f] - mu);       // m = -inf: 0
            m[f] = mn;
            float ps = 0.f;
#pragma unroll
            for (int g = 0; g < 2; ++g)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float a = __builtin_amdgcn_exp2f(fmaf(sc[8 * g + 2 * j], LOG2E, -mu));
                    const float b = __builtin_amdgcn_exp2f(fmaf(sc[8 * g + 2 * j + 1], LOG2E, -mu));
                    ps += a + b;
                    pb[f][g][j] = pack_bf2(a, b);
                }
            l[f] = l[f] * alpha + ps;
            if (__builtin_expect(__any(alpha != 1.0f), 0)) {
#pragma unroll
                for (int c = 0; c < CT; ++c)
#pragma unroll
                    for (int r = 0; r < 16; ++r) o[f][c][r] *= alpha;
            }
        });
        // k-slot (hi, e) of half g <-> key 16 g + 8 (e / 4) + 4 hi + e % 4: exactly the weights this lane holds
        const int ta = lane & 15, g1 = (lane >> 4) & 1;
        const unsigned char* vrow = blk + (4 * hi + (ta >> 2)) * (S::PPR * 16) + (ta & 1) * 8;
        const unsigned vcol = (unsigned)(((2 * g1 + ((ta & 3) >> 1)) ^ ((((ta >> 2) << 2) | hi) & S::XM)) * 16);
        each<CT>([&](auto cc) {
            constexpr int c = decltype(cc)::value;                       // (rows 8 further on: bit 1 of the swizzle turns)
            const unsigned o0 = flip<64 * c>(vcol), o1 = flip<(64 * c) ^ ((2 & S::XM) * 16)>(vcol);
#pragma unroll
            for (int g = 0; g < 2; ++g) {
                const s4 t0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)(vrow + (16 * g) * (S::PPR * 16) + o0));
                const s4 t1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)(vrow + (16 * g + 8) * (S::PPR * 16) + o1));
                const v2u a = __builtin_bit_cast(v2u, t0), b = __builtin_bit_cast(v2u, t1);
                const bf8 v = __builtin_bit_cast(bf8, (v4u{a[0], a[1], b[0], b[1]}));
#pragma unroll
                for (int f = 0; f < M; ++f)
                    o[f][c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, __builtin_bit_cast(bf8, (v4u{pb[f][g][0], pb[f][g][1], pb[f][g][2], pb[f][g][3]})),
                                                                      o[f][c], 0, 0, 0);
            }
        });
    }
};

// Copy ROWS cache rows that lie behind each other at `base` into LDS at `dst` with WAVES waves (this one is number w), 1 KiB per wave and
// instruction: piece p = 64 (w + WAVES j) + lane, row p / PPR.  Rows past `left` repeat row `left`.  base, dst, w: wave-uniform.
template <typename S, int ROWS, int WAVES>
__device__ __forceinline__ void copy_rows(const bf16_t* base, unsigned dst, int left, int w, int lane) {
    constexpr int N = ROWS * S::PPR / (64 * WAVES), PER = 64 * WAVES, RPI = PER / S::PPR;        // instructions; pieces, rows of one
    static_assert(ROWS * S::PPR % (64 * WAVES) == 0, "");
    auto piece = [&](unsigned off, const bf16_t* from, int j) {
        asm volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, %1" ::"v"(off), "s"(from), "s"(dst + (w + WAVES * j) * 1024)
                     : "memory");
    };
    auto offset = [&](int j) {
        const int p = 64 * (w + WAVES * j) + lane, row = p / S::PPR, c = p - row * S::PPR;
        return (unsigned)((min(row, left) * S::PPR + (c ^ S::swizzle(row))) * 16);
    };
    if (PER % S::PPR == 0 && RPI % 8 == 0 && left >= ROWS - 1) {
        // every instruction advances by the same rows: one offset, the rows in the base, and (8 rows) a swizzle that alternates
        const unsigned o0 = offset(0), o1 = o0 ^ (RPI % 16 ? (2 & S::XM) * 16 : 0);
#pragma unroll
        for (int j = 0; j < N; ++j) piece(j & 1 ? o1 : o0, base + (size_t)j * RPI * S::PPR * 8, j);
    } else {
#pragma unroll
        for (int j = 0; j < N; ++j) piece(offset(j), base, j);
    }
}

// A sequence's page ids, 64 at a time in a register (lane i: page 64 c + i): the key loop looks them up without a memory round trip.
struct PageIds {
    const int32_t* bt;
    int n, ids, c;
    __device__ __forceinline__ PageIds(const int32_t* table, int entries, int lane) : bt(table), n(entries), c(0) { fetch(lane); }
    __device__ __forceinline__ void fetch(int lane) { ids = bt[min(64 * c + lane, n - 1)]; }
    __device__ __forceinline__ int at(int i, int lane) {                 // i: wave-uniform
        if ((i >> 6) != c) {
            c = i >> 6;
            fetch(lane);
        }
        return __builtin_amdgcn_readlane(ids, i & 63);
    }
};

template <int DT, int CT, int M>
__global__ __launch_bounds__(NT, (Shape<DT, CT, M>::PROMPT_OCC)) void maps_prompt_kernel(MapsArgs a) {
    using S = Shape<DT, CT, M>;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int li = lane & 31, hi = lane >> 5;
    // workgroup id: an XCD's share (every 8th launched) is a run of neighbouring ids; a pool's tiles of a sequence are neighbours, last first
    const int nwg = gridDim.x, xcd = blockIdx.x & 7, share = nwg >> 3, rest = nwg & 7;
    const int id = xcd * share + min(xcd, rest) + (blockIdx.x >> 3);
    const int y = id / a.n_tiles, tix = a.n_tiles - 1 - id % a.n_tiles;
    const int pool_id = y / a.HG, h0 = pool_id * a.per + (y % a.HG) * 32, h_end = pool_id * a.per + a.per;
    const int slot = a.tiles[3 * tix], t0 = a.tiles[3 * tix + 1], ntok = a.tiles[3 * tix + 2];
    const bf16_t* pool = a.pool + (size_t)pool_id * (size_t)a.pool_stride;
    const int32_t* bt = a.block_table + (size_t)slot * a.table_stride;
    const int p_first = a.pos[t0], p_last = p_first + ntok - 1;
    const int tok = w * a.TQ + li / a.HP, head = h0 + li % a.HP;         // (li / HP < TQ)
    const bool ok = tok < ntok && head < h_end;
    const int t = t0 + (ok ? tok : 0), p_row = p_first + (ok ? tok : 0);
    const int wp_first = p_first + w * a.TQ, wp_last = min(wp_first + a.TQ - 1, p_last);      // (a wave without tokens: wp_first > p_last)
    Rows<DT, CT, M> R;
    R.start(a.q + ((size_t)t * a.H + (ok ? head : 0)) * (M * S::DIM), ok, hi);
    const unsigned lds = (unsigned)(size_t)(lds_ptr)smem;
    const int ntiles = p_last / (2 * BN) + 1;
    PageIds pages(bt, (p_last >> a.page_shift) + 1, lane);
    auto base_of = [&](int k0) {
        const int page = pages.at(k0 >> a.page_shift, lane);
        return pool + (((size_t)page << a.page_shift) + (size_t)(k0 & ((1 << a.page_shift) - 1))) * (size_t)(8 * S::PPR);
    };
    auto copy_tile = [&](int tile, int buf) {
        const int k0 = tile * 2 * BN;
        copy_rows<S, 2 * BN, NW>(base_of(k0), lds + 2 * buf * S::BLOCK, p_last - k0, w, lane);
    };
    copy_tile(0, 0);
#pragma unroll
    for (int f = 0; f < M; ++f)
#pragma unroll
        for (int s = 0; s < DT; ++s) asm volatile("" : "+v"(R.qf[f][s]));      // (complete before the loop: its waits count the copies only)
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    for (int tile = 0; tile < ntiles; ++tile) {
        const int buf = tile & 1;
        if (tile + 1 < ntiles) copy_tile(tile + 1, buf ^ 1);
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const int k0 = tile * 2 * BN + b * BN;
            if (k0 <= wp_last && wp_first <= p_last) R.block(smem + (2 * buf + b) * S::BLOCK, k0, p_row, k0 + BN - 1 > wp_first, lane);
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
    }
    if (!ok) return;                                                    // (lanes li and li + 32 leave together)
    float f;
    if (M == 2) {
        const float i1 = 1.0f / (R.l[0] + __shfl_xor(R.l[0], 32, 64)), i2 = a.lambda / (R.l[M - 1] + __shfl_xor(R.l[M - 1], 32, 64));
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < CT; ++c)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const float v = R.o[0][c][r] * i1 - R.o[M - 1][c][r] * i2;
                R.o[0][c][r] = v;
                sq += v * v;
            }
        sq += __shfl_xor(sq, 32, 64);
        f = a.out_scale / sqrtf(sq / (float)S::VDIM + a.eps);
    } else {
        f = 1.0f / (R.l[0] + __shfl_xor(R.l[0], 32, 64));
    }
    bf16_t* orow = a.out + ((size_t)t * a.H + head) * S::VDIM;
    const bf16_t* grow = a.gate ? a.gate + (size_t)t * (size_t)a.gate_stride + (size_t)head * S::VDIM : nullptr;
#pragma unroll
    for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int e = 32 * c + 8 * j + 4 * hi;
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = R.o[0][c][4 * j + r] * f;
            if (grow) {
                const Vec<4> g = ldv<4>(grow, e);
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] *= 1.0f / (1.0f + __expf(-g.v[r]));
            }
            *(v2u*)(orow + e) = v2u{pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3])};
        }
}

// One row from n partial results: src(i, f) its unnormalised output of map f, ml(i, f) its (maximum, sum); the wave's lanes walk vdim.
template <int VDIM, int M, typename FO, typename FM>
__device__ __forceinline__ void finish_row(const MapsArgs& a, int n, FO src, FM ml, size_t t, int head, int lane) {
    constexpr int EO = (VDIM + 63) / 64;
    float o[EO];
#pragma unroll
    for (int i = 0; i < EO; ++i) o[i] = 0.f;
#pragma unroll
    for (int f = 0; f < M; ++f) {
        float mx = -INFINITY, L = 0.f, acc[EO];
        for (int k = 0; k < n; ++k) mx = fmaxf(mx, ml(k, f)[0]);
#pragma unroll
        for (int i = 0; i < EO; ++i) acc[i] = 0.f;
        for (int k = 0; k < n; ++k) {
            const float e = __builtin_amdgcn_exp2f(ml(k, f)[0] - mx);    // (a part without keys: 0)
            L += e * ml(k, f)[1];
#pragma unroll
            for (int i = 0; i < EO; ++i)
                if (lane + 64 * i < VDIM) acc[i] += e * src(k, f)[lane + 64 * i];
        }
        const float s = (f == 0 ? 1.0f : -a.lambda) / L;
#pragma unroll
        for (int i = 0; i < EO; ++i) o[i] += s * acc[i];
    }
    float inv = 1.0f;
    if (M == 2) {
        float sq = 0.f;
#pragma unroll
        for (int i = 0; i < EO; ++i) sq += o[i] * o[i];
        inv = a.out_scale / sqrtf(wave_sum(sq) / (float)VDIM + a.eps);
    }
#pragma unroll
    for (int i = 0; i < EO; ++i) {
        const int e = lane + 64 * i;
        if (e >= VDIM) continue;
        float v = o[i] * inv;
        if (a.gate) v *= 1.0f / (1.0f + __expf(-bf2f(a.gate[t * (size_t)a.gate_stride + (size_t)head * VDIM + e])));
        a.out[(t * a.H + head) * (size_t)VDIM + e] = f2bf(v);
    }
}

template <int DT, int CT, int M>
__global__ __launch_bounds__(NT, (Shape<DT, CT, M>::STEP_OCC)) void maps_step_kernel(MapsArgs a) {
    using S = Shape<DT, CT, M>;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int li = lane & 31, hi = lane >> 5;
    const int y = blockIdx.y, z = blockIdx.z;
    const int pool_id = y / a.HG, h0 = pool_id * a.per + (y % a.HG) * 32, h_end = pool_id * a.per + a.per;
    const int slot = a.tiles[3 * blockIdx.x], t0 = a.tiles[3 * blockIdx.x + 1], ntok = a.tiles[3 * blockIdx.x + 2];
    const bf16_t* pool = a.pool + (size_t)pool_id * (size_t)a.pool_stride;
    const int32_t* bt = a.block_table + (size_t)slot * a.table_stride;
    const int p_first = a.pos[t0], p_last = p_first + ntok - 1;
    const int tok = li / a.HP, head = h0 + li % a.HP;
    const bool ok = tok < ntok && head < h_end;
    const int t = t0 + (ok ? tok : 0), p_row = p_first + (ok ? tok : 0);
    Rows<DT, CT, M> R;
    R.start(a.q + ((size_t)t * a.H + (ok ? head : 0)) * (M * S::DIM), ok, hi);
    const unsigned lds = (unsigned)(size_t)(lds_ptr)smem + w * S::BUFS * S::BLOCK;
    const unsigned char* mine = smem + w * S::BUFS * S::BLOCK;
    const int nT = p_last / BN + 1, stride = NW * a.Z, first = z * NW + w;
    PageIds pages(bt, (p_last >> a.page_shift) + 1, lane);
    auto copy = [&](int tile, int buf) {
        const int k0 = tile * BN, page = pages.at(k0 >> a.page_shift, lane);
        copy_rows<S, BN, 1>(pool + (((size_t)page << a.page_shift) + (size_t)(k0 & ((1 << a.page_shift) - 1))) * (size_t)(8 * S::PPR), lds + buf * S::BLOCK,
                            p_last - k0, 0, lane);
    };
    if (first < nT) copy(first, 0);
#pragma unroll
    for (int f = 0; f < M; ++f)
#pragma unroll
        for (int s = 0; s < DT; ++s) asm volatile("" : "+v"(R.qf[f][s]));
    int i = 0;
    for (int tile = first; tile < nT; tile += stride, ++i) {
        const bool more = tile + stride < nT;
        if (S::BUFS == 2 && more) {
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");           // (the other buffer has been read)
            copy(tile + stride, (i + 1) & 1);
            asm volatile("s_waitcnt vmcnt(%0)" ::"n"(S::PPR / 2) : "memory");    // this block has landed, the next one may be on its way
        } else {
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        }
        R.block(mine + (S::BUFS == 2 ? (i & 1) : 0) * S::BLOCK, tile * BN, p_row, tile * BN + BN - 1 > p_first, lane);
        if (S::BUFS == 1 && more) {
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
            copy(tile + stride, 0);
        }
    }
    // ---- merge the four waves ----
    float* so = (float*)smem;                                            // [NW][M][32][OROW]
    float* sml = (float*)(smem + S::STEP_LDS - S::ML);                   // [NW][M][32][2]
    __syncthreads();                                                     // every wave has read its last block
    if (ok) {
#pragma unroll
        for (int f = 0; f < M; ++f) {
            const float l = R.l[f] + __shfl_xor(R.l[f], 32, 64);
            const int row = (w * M + f) * 32 + li;
            if (hi == 0) {
                sml[2 * row] = R.m[f];
                sml[2 * row + 1] = l;
            }
#pragma unroll
            for (int c = 0; c < CT; ++c)
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    *(float4*)(so + row * S::OROW + 32 * c + 8 * j + 4 * hi) =
                        make_float4(R.o[f][c][4 * j], R.o[f][c][4 * j + 1], R.o[f][c][4 * j + 2], R.o[f][c][4 * j + 3]);
        }
    }
    __syncthreads();
    for (int row = w; row < 32; row += NW) {
        const int rt = row / a.HP, rh = h0 + row % a.HP;
        if (rt >= ntok || rh >= h_end) continue;                         // (wave-uniform)
        auto src = [&](int k, int f) { return so + ((k * M + f) * 32 + row) * S::OROW; };
        auto ml = [&](int k, int f) { return sml + ((k * M + f) * 32 + row) * 2; };
        if (a.Z == 1) {
            finish_row<S::VDIM, M>(a, NW, src, ml, (size_t)(t0 + rt), rh, lane);
            continue;
        }
        const size_t at = (((size_t)z * a.n_tiles + blockIdx.x) * gridDim.y + y) * 32 + row;
#pragma unroll
        for (int f = 0; f < M; ++f) {
            float mx = -INFINITY, L = 0.f;
#pragma unroll
            for (int k = 0; k < NW; ++k) mx = fmaxf(mx, ml(k, f)[0]);
            const float mu = mx == -INFINITY ? 0.f : mx;                 // (no key in this split)
            float e[NW];
#pragma unroll
            for (int k = 0; k < NW; ++k) {
                e[k] = __builtin_amdgcn_exp2f(ml(k, f)[0] - mu);
                L += e[k] * ml(k, f)[1];
            }
            if (lane == 0) {
                a.part_ml[(at * M + f) * 2] = mx;
                a.part_ml[(at * M + f) * 2 + 1] = L;
            }
            for (int c = lane; c < S::VDIM; c += 64) {
                float v = 0.f;
#pragma unroll
                for (int k = 0; k < NW; ++k) v += e[k] * src(k, f)[c];
                a.part_o[(at * M + f) * S::VDIM + c] = v;
            }
        }
    }
}

template <int VDIM, int M>
__global__ __launch_bounds__(NT) void maps_merge_kernel(MapsArgs a) {
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, y = blockIdx.y;
    const int pool_id = y / a.HG, h0 = pool_id * a.per + (y % a.HG) * 32, h_end = pool_id * a.per + a.per;
    const int t0 = a.tiles[3 * blockIdx.x + 1], ntok = a.tiles[3 * blockIdx.x + 2];
    for (int row = w; row < 32; row += NW) {
        const int rt = row / a.HP, rh = h0 + row % a.HP;
        if (rt >= ntok || rh >= h_end) continue;
        auto at = [&](int k, int f) { return ((((size_t)k * a.n_tiles + blockIdx.x) * gridDim.y + y) * 32 + row) * M + f; };
        finish_row<VDIM, M>(a, a.Z, [&](int k, int f) { return a.part_o + at(k, f) * VDIM; }, [&](int k, int f) { return a.part_ml + at(k, f) * 2; },
                            (size_t)(t0 + rt), rh, lane);
    }
}

template <int DT, int CT, int M>
int launch_maps(MapsArgs a, const int32_t* prompt_tiles, int n_prompt, const int32_t* step_tiles, int n_step, int G, hipStream_t st) {
    using S = Shape<DT, CT, M>;
    const int gy = G * a.HG;
    if (n_prompt > 0) {
        a.tiles = prompt_tiles;
        a.n_tiles = n_prompt;
        if (S::PROMPT_LDS > 64 * 1024) {
            const hipError_t e = hipFuncSetAttribute((const void*)maps_prompt_kernel<DT, CT, M>, hipFuncAttributeMaxDynamicSharedMemorySize, S::PROMPT_LDS);
            QSV_REQUIRE(e == hipSuccess, "qsv_maps_attention: %s", hipGetErrorString(e));
        }
        hipLaunchKernelGGL((maps_prompt_kernel<DT, CT, M>), dim3(n_prompt * gy), dim3(NT), S::PROMPT_LDS, st, a);
        const int rc = qsv_launch_status("qsv_maps_attention (prompt)");
        if (rc != QSV_OK) return rc;
    }
    if (n_step > 0) {
        a.tiles = step_tiles;
        a.n_tiles = n_step;
        if (S::STEP_LDS > 64 * 1024) {
            const hipError_t e = hipFuncSetAttribute((const void*)maps_step_kernel<DT, CT, M>, hipFuncAttributeMaxDynamicSharedMemorySize, S::STEP_LDS);
            QSV_REQUIRE(e == hipSuccess, "qsv_maps_attention: %s", hipGetErrorString(e));
        }
        hipLaunchKernelGGL((maps_step_kernel<DT, CT, M>), dim3(n_step, gy, a.Z), dim3(NT), S::STEP_LDS, st, a);
        const int rc = qsv_launch_status("qsv_maps_attention (step)");
        if (rc != QSV_OK) return rc;
        if (a.Z > 1) hipLaunchKernelGGL((maps_merge_kernel<S::VDIM, M>), dim3(n_step, gy), dim3(NT), 0, st, a);
    }
    return qsv_launch_status("qsv_maps_attention");
}
int head_slots(int per) {
    int hp = 1;
    while (hp < per && hp < 32) hp <<= 1;
    return hp;
}
#define QSV_MAPS_SHAPES(F) F(1, 1, 2) F(2, 1, 2) F(2, 2, 2) F(3, 3, 2) F(4, 2, 2) F(4, 4, 2) F(6, 3, 2) F(8, 4, 2) F(2, 1, 1) F(4, 2, 1) F(6, 3, 1) F(8, 4, 1)
}  // namespace

// 1 if the matrix-core kernels take these sizes (bfloat16 storage, pages a power of two from 64 on), else 0.
extern "C" int qsv_maps_attention_ok(int dim, int vdim, int maps, int page, int dtype) {
    if (dtype != QSV_BF16 || page < 2 * BN || (page & (page - 1))) return 0;
#define QSV_MAPS_OK(DT, CT, M) \
    if (dim == 16 * DT && vdim == 32 * CT && maps == M) return 1;
    QSV_MAPS_SHAPES(QSV_MAPS_OK)
#undef QSV_MAPS_OK
    return 0;
}
// Tokens of one sequence a wave (step tiles) serves for `heads` heads per pool; prompt tiles hold up to four times as many.
extern "C" int qsv_maps_attention_tile_tokens(int heads_per_pool) { return heads_per_pool > 0 ? 32 / head_slots(heads_per_pool) : 0; }
// Rows of the step tiles' partial results per (tile, pool): 32 per head group of 32.
extern "C" int qsv_maps_attention_head_groups(int heads_per_pool) { return heads_per_pool > 0 ? (heads_per_pool + 31) / 32 : 0; }

extern "C" int qsv_maps_attention(void* out, const void* q, const void* pool, const int32_t* block_table, int table_stride, const int32_t* pos,
                                  const int32_t* prompt_tiles, int n_prompt, const int32_t* step_tiles, int n_step, int H, int G, int dim,
                                  int vdim, int maps, int page, int64_t pool_stride, float lambda, float out_scale, float eps, const void* gate,
                                  int64_t gate_stride, int key_splits, float* part_o, float* part_ml, void* stream) {
    QSV_REQUIRE(out && q && pool && block_table && pos && n_prompt >= 0 && n_step >= 0 && (!n_prompt || prompt_tiles) && (!n_step || step_tiles),
                "qsv_maps_attention: null argument");
    QSV_REQUIRE(H > 0 && G > 0 && H % G == 0 && table_stride > 0 && pool_stride >= 0, "qsv_maps_attention: %d heads over %d", H, G);
    QSV_REQUIRE(qsv_maps_attention_ok(dim, vdim, maps, page, QSV_BF16), "qsv_maps_attention: %d maps of %d over values of %d, pages of %d", maps, dim, vdim,
                page);
    QSV_REQUIRE((uintptr_t)q % 16 == 0 && (uintptr_t)pool % 16 == 0 && pool_stride % 8 == 0 && (uintptr_t)out % 8 == 0, "qsv_maps_attention: unaligned");
    QSV_REQUIRE(!gate || (gate_stride >= (int64_t)H * vdim && gate_stride % 4 == 0 && (uintptr_t)gate % 8 == 0), "qsv_maps_attention: gate rows");
    QSV_REQUIRE(key_splits >= 1 && key_splits <= 64 && (key_splits == 1 || !n_step || (part_o && part_ml)), "qsv_maps_attention: key splits without workspace");
    const int per = H / G, HG = (per + 31) / 32;
    QSV_REQUIRE((int64_t)n_prompt * G * HG < (1ll << 31) && G * HG <= 65535, "qsv_maps_attention: too many tiles");
    MapsArgs a = {(bf16_t*)out, (const bf16_t*)q, (const bf16_t*)pool, (const bf16_t*)gate, block_table, pos, nullptr, part_o, part_ml, pool_stride,
                  gate_stride, table_stride, 0, H, per, __builtin_ctz(page), head_slots(per), 32 / head_slots(per), HG, key_splits, lambda, out_scale, eps};
#define QSV_MAPS_RUN(DT, CT, M)                      \
    if (dim == 16 * DT && vdim == 32 * CT && maps == M) \
        return launch_maps<DT, CT, M>(a, prompt_tiles, n_prompt, step_tiles, n_step, G, (hipStream_t)stream);
    QSV_MAPS_SHAPES(QSV_MAPS_RUN)
#undef QSV_MAPS_RUN
    return QSV_EINVAL;
}

extern "C" int qsv_conv_heads_cache(void* q, void* pool, int64_t pool_rows, const void* proj, int64_t stride, const float* w, int taps, float* hist,
                                    const int32_t* run_off, const int32_t* state_rd, const int32_t* state_wr, const int64_t* slot,
                                    const int32_t* pos, int q_channels, int kv_heads, int key_width, int vdim, float scale, float temp_coef,
                                    double temp_every, int n, int dtype, void* stream) {
    QSV_REQUIRE(q && proj && w && run_off && state_rd && state_wr && pos, "qsv_conv_heads_cache: null argument");
    QSV_REQUIRE(n >= 0 && taps >= 1 && q_channels > 0 && kv_heads >= 0 && (taps == 1 || hist), "qsv_conv_heads_cache: %d taps without a history", taps);
    QSV_REQUIRE(!kv_heads || (pool && slot && key_width > 0 && vdim > 0), "qsv_conv_heads_cache: keys and values without a cache");
    ConvHeads a = {w, hist, run_off, state_rd, state_wr, pos, slot, stride, pool_rows, taps - 1, 0, q_channels, key_width > 0 ? key_width : 1,
                   vdim > 0 ? vdim : 1, kv_heads * key_width, scale, temp_coef, temp_every};
    a.C = q_channels + kv_heads * (key_width + vdim);
    QSV_REQUIRE(stride >= a.C, "qsv_conv_heads_cache: %d channels in rows of %lld", a.C, (long long)stride);
    QSV_REQUIRE(!(temp_every < 0.0), "qsv_conv_heads_cache: temperature step %g", temp_every);
    if (n == 0) return QSV_OK;
    const size_t es = dtype == QSV_F32 ? 4 : 2;
    auto al = [](const void* p, size_t size) { return (uintptr_t)p % (4 * size) == 0; };
    const bool vec = q_channels % 4 == 0 && stride % 4 == 0 && (!kv_heads || (key_width % 4 == 0 && vdim % 4 == 0)) && al(q, es) && al(proj, es) && al(w, 4) &&
                     al(hist, 4) && (!kv_heads || al(pool, es));
    if (vec && n >= 2 * TB && taps >= 2 && taps <= 4) {
        const dim3 grid((n + TB - 1) / TB, (a.C / 4 + NT - 1) / NT);
#define QSV_CHR(P)                                                                                                                     \
    QSV_DISPATCH(dtype, "qsv_conv_heads_cache",                                                                                        \
                 hipLaunchKernelGGL((conv_heads_rows_kernel<T, P>), grid, dim3(NT), 0, (hipStream_t)stream, (T*)q, (T*)pool, (const T*)proj, a, n))
        if (taps == 2) QSV_CHR(1);
        else if (taps == 3) QSV_CHR(2);
        else QSV_CHR(3);
#undef QSV_CHR
        return qsv_launch_status("qsv_conv_heads_cache");
    }
#define QSV_CH(V)                                                                                                                      \
    QSV_DISPATCH(dtype, "qsv_conv_heads_cache",                                                                                        \
                 hipLaunchKernelGGL((conv_heads_kernel<T, V>), dim3(n, (a.C / V + NT - 1) / NT), dim3(NT), 0, (hipStream_t)stream, (T*)q, (T*)pool, \
                                    (const T*)proj, a))
    if (vec) QSV_CH(4);
    else QSV_CH(1);
#undef QSV_CH
    return qsv_launch_status("qsv_conv_heads_cache");
}

extern "C" int qsv_diff_attention(void* out, const void* q, const void* pool, const int32_t* block_table, int table_stride, const int32_t* seq,
                                  const int32_t* pos, int n, int H, int G, int dim, int vdim, int page, int64_t pool_stride, float lambda,
                                  float out_scale, float eps, const void* gate, int64_t gate_stride, int dtype, void* stream) {
    QSV_REQUIRE(out && q && pool && block_table && seq && pos, "qsv_diff_attention: null argument");
    QSV_REQUIRE(n >= 0 && H > 0 && G > 0 && H % G == 0, "qsv_diff_attention: %d heads over %d", H, G);
    QSV_REQUIRE(dim > 0 && dim <= 512 && vdim > 0 && vdim <= 1024 && page > 0 && table_stride > 0 && pool_stride >= 0,
                "qsv_diff_attention: heads of %d (at most 512) and %d (at most 1024) elements", dim, vdim);
    QSV_REQUIRE(!gate || gate_stride >= (int64_t)H * vdim, "qsv_diff_attention: gate rows of %lld", (long long)gate_stride);
    if (n == 0) return QSV_OK;
    QSV_REQUIRE((int64_t)n * H < (1ll << 31), "qsv_diff_attention: too many (token, head) pairs");
#define QSV_DA(EK, EV)                                                                                                                 \
    QSV_DISPATCH(dtype, "qsv_diff_attention",                                                                                          \
                 hipLaunchKernelGGL((diff_attention_wave_kernel<T, EK, EV>), dim3(n * H), dim3(NT), 0, (hipStream_t)stream, (T*)out, (const T*)q, \
                                    (const T*)pool, block_table, table_stride, seq, pos, H, H / G, dim, vdim, page, pool_stride, lambda, out_scale, \
                                    eps, (const T*)gate, gate_stride))
    if (dim <= 64 && vdim <= 64) QSV_DA(1, 1);
    else if (dim <= 64 && vdim <= 128) QSV_DA(1, 2);
    else if (dim <= 128 && vdim <= 256) QSV_DA(2, 4);
    else if (dim <= 256 && vdim <= 512) QSV_DA(4, 8);
    else QSV_DA(8, 16);
#undef QSV_DA
    return qsv_launch_status("qsv_diff_attention");
}
