// serve_talking.hip -- talking-heads attention over the paged cache: every head's softmax weights are mixed with the other heads'
// before they meet the values,  out_h = sum_j (sum_g talk[h, g] w_g(j)) v_kv(h)(j).
//
// Two forms.  Weights mixed before the sum ("two passes", up to 32 heads of up to 128 elements, bfloat16): the first launch finds every
// head's maximum and sum, the second computes the scores again, normalises, mixes the heads' weights on the matrix cores and
// multiplies each head's own values.  Its result is final but for the sum over key splits.
//
// Any sizes: the mix is linear, so it can come AFTER the sum over the keys, at the price of every head summing every pool's values:
//   A[g, k] = sum_j w_g(j) v_k(j)           out_h = gate_h sum_g talk[h, g] A[g, kv(h)]
// A is float; the last kernel merges the key splits, normalises, mixes and gates in one pass.
//
// Scores: (qf . k), qf already scaled; cap > 0: cap tanh(. / cap).  With 0 < cap <= FIXED_CAP every score lies in [-cap, cap] and `cap`
// itself serves as the softmax's maximum: no running maximum, no rescaling (e^(-2 cap) stays a normal float).
//
// Cache: per key / value head one pool of rows [v (vdim) | k (dim)].
#include "serve_common.h"

namespace {
constexpr int NT = 256;
constexpr int NW = NT / 64;
constexpr int KG = 4;              // wave kernel: keys per softmax update
constexpr float FIXED_CAP = 40.f;

// ---- wave kernel: any sizes, both storage types -----------------------------------------------------------------------------------
// Workgroup = (token, head) x one value pool; wave w takes keys KG (w + 4 n) .., lanes over a row's elements.
template <typename T, int EPL>
__global__ __launch_bounds__(NT) void talking_wave_kernel(float* __restrict__ part_o, const float* __restrict__ qf, const T* __restrict__ pool,
                                                          const int32_t* __restrict__ block_table, int table_stride,
                                                          const int32_t* __restrict__ seq, const int32_t* __restrict__ pos, int window,
                                                          int H, int G, int dim, int vdim, int page, int64_t pool_stride, float cap) {
    __shared__ float s_m[NW], s_l[NW];
    __shared__ float s_acc[NW][64 * EPL];
    const size_t t = blockIdx.x / H;
    const int h = blockIdx.x % H, vp = blockIdx.y, per = H / G, R = vdim + dim;
    const T* kpool = pool + (size_t)(h / per) * (size_t)pool_stride + vdim;
    const T* vpool = pool + (size_t)vp * (size_t)pool_stride;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int p = pos[t];
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    const int32_t* bt = block_table + (size_t)seq[t] * table_stride;
    const float* qrow = qf + (t * H + h) * (size_t)dim;
    float q[EPL], acc[EPL];
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
        const int e = lane + 64 * i;
        q[i] = e < dim ? qrow[e] : 0.f;
        acc[i] = 0.f;
    }
    float m = -INFINITY, l = 0.f;
    for (int j0 = lo + w * KG; j0 <= p; j0 += NW * KG) {
        float c[KG][EPL], s[KG];
#pragma unroll
        for (int k = 0; k < KG; ++k) {
            const int j = j0 + k, jj = min(j, p);
            const size_t row = ((size_t)bt[jj / page] * page + (size_t)(jj % page)) * (size_t)R;
            float d = 0.f;
#pragma unroll
            for (int i = 0; i < EPL; ++i) {
                const int e = lane + 64 * i;
                d += q[i] * (e < dim ? ld(kpool, row + e) : 0.f);
                c[k][i] = e < vdim ? ld(vpool, row + e) : 0.f;
            }
            d = wave_sum(d);
            if (cap > 0.f) d = cap * tanhf(d / cap);
            s[k] = j <= p ? d : -INFINITY;
        }
        float mx = m;
#pragma unroll
        for (int k = 0; k < KG; ++k) mx = fmaxf(mx, s[k]);
        const float alpha = expf(m - mx);
        float pk[KG], ps = 0.f;
#pragma unroll
        for (int k = 0; k < KG; ++k) {
            pk[k] = expf(s[k] - mx);
            ps += pk[k];
        }
        l = l * alpha + ps;
        m = mx;
#pragma unroll
        for (int i = 0; i < EPL; ++i) {
            float a = acc[i] * alpha;
#pragma unroll
            for (int k = 0; k < KG; ++k) a += pk[k] * c[k][i];
            acc[i] = a;
        }
    }
    if (lane == 0) {
        s_m[w] = m;
        s_l[w] = l;
    }
#pragma unroll
    for (int i = 0; i < EPL; ++i) s_acc[w][lane + 64 * i] = acc[i];
    __syncthreads();
    float M = s_m[0];
#pragma unroll
    for (int k = 1; k < NW; ++k) M = fmaxf(M, s_m[k]);
    float f[NW], L = 0.f;
#pragma unroll
    for (int k = 0; k < NW; ++k) {
        f[k] = expf(s_m[k] - M);                   // a wave without keys has m = -inf: factor 0
        L += f[k] * s_l[k];
    }
    const float invL = 1.0f / L;
    float* o = part_o + ((t * H + h) * (size_t)G + vp) * vdim;
    for (int e = threadIdx.x; e < vdim; e += NT) {
        float a = 0.f;
#pragma unroll
        for (int k = 0; k < NW; ++k) a += f[k] * s_acc[k][e];
        o[e] = a * invL;
    }
}

// ---- matrix-core kernel (bfloat16 storage) -----------------------------------------------------------------------------------------
// A workgroup of four waves serves a tile of consecutive tokens of one sequence, for the heads of KP neighbouring key pools and the
// values of NP neighbouring pools.  A wave owns 16 query rows = TQ tokens x HP head slots.  Keys are contracted over the KP pools' rows laid
// side by side (KP dim elements, the query zero outside its own pool's part): decoding takes KP so that the 16 rows are heads of one
// token and a key is staged once for all of them; prompt tiles take KP = 1.  Tiles of 32 keys are staged in LDS, keys and values
// row-major; values are transposed as they are read (ds_read_b64_tr_b16).  S^T = K Q^T leaves a lane eight scores of its own row, which
// are the B operand of O^T = V^T P^T as they stand.  Few tokens per tile: the waves split the key tiles and merge through LDS.
typedef float v4f __attribute__((ext_vector_type(4)));
typedef __bf16 bf8 __attribute__((ext_vector_type(8)));
typedef unsigned int v4u __attribute__((ext_vector_type(4)));
typedef unsigned int v2u __attribute__((ext_vector_type(2)));
typedef short s4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s4* lds_s4;
constexpr int BN = 32;             // keys per tile

__device__ __forceinline__ unsigned pack_bf2(float a, float b) { return (unsigned)f2bf(a) | ((unsigned)f2bf(b) << 16); }
__host__ __device__ constexpr int k_row(int dt) { return 32 * dt + 8; }                       // LDS row strides (elements): the 16 rows of a
__host__ __device__ inline int v_row(int cols) { return ((cols + 127) & ~127) + 16; }          // read spread over all banks

// DT: 32-element steps of the key contraction (KP dim <= 32 DT); CT: 16-column tiles of the values (NP vdim <= 16 CT).
template <int DT, int CT>
__global__ __launch_bounds__(NT, (DT >= 16 ? 1 : 2)) void talking_mfma_kernel(
    float* __restrict__ part_o, float* __restrict__ part_ml, const float* __restrict__ qf, const bf16_t* __restrict__ pool,
    const int32_t* __restrict__ block_table, int table_stride, const int32_t* __restrict__ pos, const int32_t* __restrict__ tiles,
    int window, int H, int G, int dim, int vdim, int page, int64_t pool_stride, float cap, int KP, int NP, int HP, int TQ, int n_tokens) {
    constexpr int KS = k_row(DT), NCK = DT / 2, NCV = CT / 4;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int R = vdim + dim, per = H / G;
    const int VS = v_row(NP * vdim);
    bf16_t* Ks = (bf16_t*)smem;                          // [BN][KS]
    bf16_t* Vs = Ks + BN * KS;                           // [BN][VS]
    float* scratch = (float*)smem;                       // merge phase

    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
    const int col = lane & 15, g4 = lane >> 4;
    const int slot = tiles[3 * blockIdx.x], t0 = tiles[3 * blockIdx.x + 1], ntok = tiles[3 * blockIdx.x + 2];
    // blockIdx.y = (key group, head group of 16 within it, value group)
    const int vg_n = (G + NP - 1) / NP, hg_n = (KP * per + 15) / 16;
    const int vg = blockIdx.y % vg_n, hg = (blockIdx.y / vg_n) % hg_n, kg = blockIdx.y / (vg_n * hg_n);
    const int kp0 = kg * KP, v0 = vg * NP, np = min(NP, G - v0);
    const int h0 = kp0 * per + hg * 16, h_end = (kp0 + KP) * per;
    const int32_t* bt = block_table + (size_t)slot * table_stride;
    const int cols = np * vdim;

    const int NG = (ntok + TQ - 1) / TQ;                 // 1 .. 4 row groups
    const int S = NW / NG;
    const bool active = w < NG * S;
    const int grp = active ? w % NG : 0, sp = active ? w / NG : 0;
    const int tok_in = grp * TQ + col / HP;
    const int head = h0 + col % HP;
    const bool row_ok = active && tok_in < ntok && head < h_end;
    const int t = t0 + (tok_in < ntok ? tok_in : 0);
    const int p_row = pos[t];
    const int lo_row = window > 0 ? max(0, p_row - window + 1) : 0;
    const int p_first = pos[t0], p_last = pos[t0 + ntok - 1];
    const int kstart = (window > 0 ? max(0, p_first - window + 1) : 0) / BN * BN;
    const int nT = (p_last - kstart) / BN + 1;
    const int gt_first = min(grp * TQ, ntok - 1), gt_last = min(grp * TQ + TQ - 1, ntok - 1);
    const int wp_first = p_first + gt_first, wp_last = p_first + gt_last;
    const int wlo = window > 0 ? max(0, wp_first - window + 1) : 0, wlo_last = window > 0 ? max(0, wp_last - window + 1) : 0;

    // query fragments: the 8 elements 32 s + 8 g4 of the row laid over the KP pools (dim % 8 == 0: a piece lies in one pool)
    v4u qfrag[DT];
    {
        const int own = row_ok ? (head / per - kp0) * dim : 0;
        const float* qrow = qf + ((size_t)t * H + (row_ok ? head : 0)) * (size_t)dim;
#pragma unroll
        for (int s = 0; s < DT; ++s) {
            const int e0 = 32 * s + 8 * g4 - own;
            float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
            if (row_ok && e0 >= 0 && e0 < dim) {
                a = *(const float4*)(qrow + e0);
                b = *(const float4*)(qrow + e0 + 4);
            }
            qfrag[s] = v4u{pack_bf2(a.x, a.y), pack_bf2(a.z, a.w), pack_bf2(b.x, b.y), pack_bf2(b.z, b.w)};
        }
    }
    const int s_n = (KP * dim + 31) / 32;
    v4f oacc[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) oacc[c] = v4f{0.f, 0.f, 0.f, 0.f};
    const bool fixed = cap > 0.f && cap <= FIXED_CAP;
    float m = fixed ? cap : -INFINITY, l = 0.f;
    const float c_in = cap > 0.f ? 2.0f * 1.4426950408889634f / cap : 0.f;        // tanh(s / cap) = 1 - 2 / (2^(c_in s) + 1)

    // staging: thread's 16-byte pieces of a tile's keys (row-major over the KP pools) and values (over the np pools)
    const int pk_n = KP * dim / 8, pv_n = cols / 8;
    int k_lds[NCK], v_lds[NCV];
    int64_t k_off[NCK], v_off[NCV];
#pragma unroll
    for (int i = 0; i < NCK; ++i) {
        const int q = tid + NT * i, row = q / pk_n, e = (q - row * pk_n) * 8;
        k_lds[i] = row < BN ? row * KS + e : -1;
        k_off[i] = (int64_t)(kp0 + e / dim) * pool_stride + (int64_t)row * R + vdim + e % dim;
    }
#pragma unroll
    for (int i = 0; i < NCV; ++i) {
        const int q = tid + NT * i, row = q / pv_n, e = (q - row * pv_n) * 8;
        v_lds[i] = row < BN ? row * VS + e : -1;
        v_off[i] = (int64_t)(v0 + e / vdim) * pool_stride + (int64_t)row * R + e % vdim;
    }
    v4u kst[NCK], vst[NCV];
    auto issue = [&](int tile) {
        const int k0 = kstart + tile * BN;
        const bf16_t* base = pool + ((size_t)bt[k0 / page] * page + (size_t)(k0 % page)) * (size_t)R;
        const int left = p_last - k0;                    // rows past the tile's last position become zeros
#pragma unroll
        for (int i = 0; i < NCK; ++i) {
            kst[i] = v4u{0u, 0u, 0u, 0u};
            if (k_lds[i] >= 0 && k_lds[i] / KS <= left) kst[i] = *(const v4u*)(base + k_off[i]);
        }
#pragma unroll
        for (int i = 0; i < NCV; ++i) {
            vst[i] = v4u{0u, 0u, 0u, 0u};
            if (v_lds[i] >= 0 && v_lds[i] / VS <= left) vst[i] = *(const v4u*)(base + v_off[i]);
        }
    };
    if (KP * dim < 32 * s_n)                             // the contraction's padding must hold numbers (the query is zero there)
        for (int i = tid; i < BN * (32 * s_n - KP * dim); i += NT) {
            const int n = 32 * s_n - KP * dim;
            Ks[(i / n) * KS + KP * dim + i % n] = 0;
        }
    const int Z = gridDim.z, z = blockIdx.z;
    int ti = 0;
    if (z < nT) issue(z);
    for (int tile = z; tile < nT; tile += Z, ++ti) {
        const int k0 = kstart + tile * BN;
        __syncthreads();                                 // the previous tile has been read
#pragma unroll
        for (int i = 0; i < NCK; ++i)
            if (k_lds[i] >= 0) *(v4u*)(Ks + k_lds[i]) = kst[i];
#pragma unroll
        for (int i = 0; i < NCV; ++i)
            if (v_lds[i] >= 0) *(v4u*)(Vs + v_lds[i]) = vst[i];
        __syncthreads();
        if (tile + Z < nT) issue(tile + Z);
        if (!active || (ti % S) != sp || k0 > wp_last || k0 + BN - 1 < wlo) continue;      // (wave-uniform)
        v4f sacc[2] = {v4f{0.f, 0.f, 0.f, 0.f}, v4f{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int s = 0; s < DT; ++s) {
            if (s >= s_n) continue;
#pragma unroll
            for (int mt = 0; mt < 2; ++mt) {
                const v4u a = *(const v4u*)(Ks + (16 * mt + col) * KS + 32 * s + 8 * g4);
                sacc[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf8, a), __builtin_bit_cast(bf8, qfrag[s]),
                                                                   sacc[mt], 0, 0, 0);
            }
        }
        // this lane: keys k0 + 16 mt + 4 g4 + r of its row
        const bool whole = k0 + BN - 1 <= wp_first && k0 >= wlo_last;   // (wave-uniform) every row sees every key of the tile
        if (fixed) {
            // e^(cap tanh - cap) = 2^(-2 cap log2(e) / (2^(c_in s) + 1)); s -> +inf: the fraction goes to 0, -inf: to 1
            const float c_out = -2.0f * 1.4426950408889634f * cap;
#pragma unroll
            for (int mt = 0; mt < 2; ++mt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int key = k0 + 16 * mt + 4 * g4 + r;
                    const float e = __builtin_amdgcn_exp2f(c_in * sacc[mt][r]);
                    float pr = __builtin_amdgcn_exp2f(c_out * __builtin_amdgcn_rcpf(e + 1.0f));
                    if (!whole && !(key <= p_row && key >= lo_row)) pr = 0.f;
                    sacc[mt][r] = pr;
                    l += pr;
                }
        } else {
            float tmax = -INFINITY;
#pragma unroll
            for (int mt = 0; mt < 2; ++mt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int key = k0 + 16 * mt + 4 * g4 + r;
                    float s = sacc[mt][r];
                    if (cap > 0.f) s = cap - 2.0f * cap * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(c_in * s) + 1.0f);
                    sacc[mt][r] = key <= p_row && key >= lo_row ? s : -INFINITY;
                    tmax = fmaxf(tmax, sacc[mt][r]);
                }
            tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
            tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
            const float mnew = fmaxf(m, tmax), msafe = mnew == -INFINITY ? 0.f : mnew;
            const float alpha = __expf(m - msafe);
            float psum = 0.f;
#pragma unroll
            for (int mt = 0; mt < 2; ++mt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    sacc[mt][r] = __expf(sacc[mt][r] - msafe);
                    psum += sacc[mt][r];
                }
            l = l * alpha + psum;
            m = mnew;
            if (__any(alpha != 1.0f)) {
#pragma unroll
                for (int c = 0; c < CT; ++c) oacc[c] *= alpha;
            }
        }
        // k-slot (g4, e) <-> key 16 (e / 4) + 4 g4 + e % 4: this lane's eight weights
        const bf8 pb = __builtin_bit_cast(bf8, (v4u{pack_bf2(sacc[0][0], sacc[0][1]), pack_bf2(sacc[0][2], sacc[0][3]),
                                                    pack_bf2(sacc[1][0], sacc[1][1]), pack_bf2(sacc[1][2], sacc[1][3])}));
        // transpose read: lane a of a 16-lane group names the piece (key 4 g4 + a / 4, columns 4 (a % 4) ..) and receives column a of the
        // group's four keys
        const bf16_t* vrow = Vs + (4 * g4 + (col >> 2)) * VS + 4 * (col & 3);
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            if (16 * c >= cols) continue;                // (uniform)
            const s4 a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)(vrow + 16 * c));
            const s4 a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)(vrow + 16 * c + 16 * VS));
            const v2u u0 = __builtin_bit_cast(v2u, a0), u1 = __builtin_bit_cast(v2u, a1);
            oacc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf8, (v4u{u0[0], u0[1], u1[0], u1[1]})), pb, oacc[c], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);

    // ---- merge the key splits (waves grp + NG s, s = 1 .. S - 1, into wave grp) ----
    if (S > 1) {                                         // (block-uniform)
        __syncthreads();                                 // the last tile has been read: LDS becomes scratch
        float* ml = scratch + NW * 8 * 64 * 4;           // [NW][64][2], behind the accumulator exchange area
        if (active && sp > 0) {
            ml[(w * 64 + lane) * 2] = m;
            ml[(w * 64 + lane) * 2 + 1] = l;
        }
        __syncthreads();
        float f[NW];
#pragma unroll
        for (int s = 0; s < NW; ++s) f[s] = 0.f;
        if (active && sp == 0) {
            float M = m;
            for (int s = 1; s < S; ++s) M = fmaxf(M, ml[((grp + NG * s) * 64 + lane) * 2]);
            const float Ms = M == -INFINITY ? 0.f : M;
            f[0] = __expf(m - Ms);
            float L = f[0] * l;
            for (int s = 1; s < S; ++s) {
                f[s] = __expf(ml[((grp + NG * s) * 64 + lane) * 2] - Ms);
                L += f[s] * ml[((grp + NG * s) * 64 + lane) * 2 + 1];
            }
            l = L;
            m = M;
        }
        constexpr int MB = CT < 8 ? CT : 8;
#pragma unroll
        for (int c0 = 0; c0 < CT; c0 += MB) {
            __syncthreads();
            if (active && sp > 0) {
#pragma unroll
                for (int j = 0; j < MB; ++j)
                    if (c0 + j < CT) *(v4f*)(scratch + ((w * MB + j) * 64 + lane) * 4) = oacc[c0 + j];
            }
            __syncthreads();
            if (active && sp == 0) {
#pragma unroll
                for (int j = 0; j < MB; ++j)
                    if (c0 + j < CT) {
                        v4f a = oacc[c0 + j] * f[0];
                        for (int s = 1; s < S; ++s) a += *(const v4f*)(scratch + (((grp + NG * s) * MB + j) * 64 + lane) * 4) * f[s];
                        oacc[c0 + j] = a;
                    }
            }
        }
    }
    if (!row_ok || sp != 0) return;
    const size_t rowi = ((size_t)z * n_tokens + t) * H + head;
    if (g4 == 0 && vg == 0) {
        part_ml[rowi * 2] = m;
        part_ml[rowi * 2 + 1] = l;
    }
    float* po = part_o + (rowi * (size_t)G + v0) * vdim;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        const int c0 = 16 * c + 4 * g4;
        if (c0 < cols) *(v4f*)(po + c0) = oacc[c];       // cols % 8 == 0: four values are inside or outside as a whole
    }
}

// ---- merge of the key splits, normalisation, head mix, output gate --------------------------------------------------------------------
// out[t, h] = sigmoid(gate[t, h]) sum_g talk[h, g] sum_z f(z, g) A[z, t, g, kv(h)],  f = e^(m_z - M) / sum_z e^(m_z - M) l_z (part_ml NULL:
// one split, already normalised).  Workgroup = token; dynamic LDS: Z H floats of f, then (H) gates.
template <typename T>
__global__ __launch_bounds__(NT) void talking_mix_kernel(T* __restrict__ out, const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                         const T* __restrict__ talk, const T* __restrict__ gate, int64_t gate_stride,
                                                         int Z, int n_tokens, int H, int G, int vdim) {
    extern __shared__ float sm[];
    float* f = sm;                                       // [Z][H]
    float* gs = sm + Z * H;                              // [H]
    float* tk = gs + H;                                  // [H][H]: talk
    const size_t t = blockIdx.x;
    for (int g = threadIdx.x; g < H; g += NT) {
        if (part_ml) {
            float M = -INFINITY, L = 0.f;
            for (int z = 0; z < Z; ++z) M = fmaxf(M, part_ml[(((size_t)z * n_tokens + t) * H + g) * 2]);
            for (int z = 0; z < Z; ++z) {
                const float* ml = part_ml + (((size_t)z * n_tokens + t) * H + g) * 2;
                L += expf(ml[0] - M) * ml[1];
            }
            for (int z = 0; z < Z; ++z) f[z * H + g] = expf(part_ml[(((size_t)z * n_tokens + t) * H + g) * 2] - M) / L;
        } else {
            f[g] = 1.0f;
        }
        gs[g] = gate ? 1.0f / (1.0f + expf(-ld(gate, t * gate_stride + g))) : 1.0f;
    }
    for (int i = threadIdx.x; i < H * H; i += NT) tk[i] = ld(talk, i);
    __syncthreads();
    const int per = H / G;
    // a thread owns column (k, c) of A and the `per` heads that read pool k, eight at a time
    for (int i = threadIdx.x; i < G * vdim; i += NT) {
        const int k = i / vdim, c = i - k * vdim;
        for (int h0 = 0; h0 < per; h0 += 8) {
            float a[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            for (int z = 0; z < Z; ++z)
                for (int g = 0; g < H; ++g) {
                    const float v = part_o[((((size_t)z * n_tokens + t) * H + g) * (size_t)G + k) * vdim + c] * f[z * H + g];
#pragma unroll
                    for (int j = 0; j < 8; ++j)
                        if (h0 + j < per) a[j] += tk[(k * per + h0 + j) * H + g] * v;
                }
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (h0 + j < per) {
                    const int h = k * per + h0 + j;
                    st(out, (t * H + h) * (size_t)vdim + c, a[j] * gs[h]);
                }
        }
    }
}

// ---- two passes: statistics, then mixed weights times values (matrix cores, bfloat16 storage) ----------------------------------------
// A workgroup of eight waves serves a tile of up to 16 consecutive tokens of one sequence and ALL heads; wave w owns heads w HW .. +HW - 1.
// Tiles of 32 keys; per tile
//   scores   S^T = K Q^T per head, 16 keys at a time: A = key rows straight from the cache (registers, shared by the wave's heads of one
//            pool; the next 16 rows are requested before the exponentials of these), B = the head's queries (registers)
//   weights  e^(score) / sum from the first pass's (maximum, sum), as float16 times 2^10, to LDS as [key][token][head]
//   mix      wave w takes four keys: talk [H x H] (A) times the weights of 16 tokens (B, contraction over the heads), result as
//            bfloat16 to LDS as [head][token][key]
//   values   O^T += V^T W^T per head: B = the mixed weights, A = the wave's value tile - copied straight into LDS of the wave's own
//            while the scores are computed, transposed as it is read
// two barriers a tile.  MODE 1 (first pass): scores and sums only, no LDS; with `scores` it also leaves the scores (in units of log 2,
// invisible pairs -inf) for the second pass, which then (MODE 2) reads neither queries nor keys: steps of few tokens, whose cost is
// reading the cache.
typedef _Float16 h8 __attribute__((ext_vector_type(8)));
typedef _Float16 h4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(1))) const void* gptr_t;
typedef __attribute__((address_space(3))) void* lptr_t;
constexpr int TT = 16;             // tokens of a tile
constexpr int TW = 8;              // waves
constexpr float LOG2E = 1.4426950408889634f;
__host__ __device__ constexpr int two_pass_gk(int hw) { return TW * hw > 16 ? 32 : 16; }     // heads the mix contracts over, padded
__host__ __device__ constexpr int two_pass_lds(int hw, int dt) {
    return TW * dt * 2048 + 2 * (BN * TT * two_pass_gk(hw) + two_pass_gk(hw) * TT * BN);
}

template <int HW, int DT, int MODE>
__global__ __launch_bounds__(64 * TW, 2) void talking_two_pass_kernel(
    bf16_t* __restrict__ out, float* __restrict__ part_o, float* __restrict__ part_ml, int Z1, const float* __restrict__ qf,
    const bf16_t* __restrict__ pool, const int32_t* __restrict__ block_table, int table_stride, const int32_t* __restrict__ pos,
    const int32_t* __restrict__ tiles, int window, int H, int G, int dim, int page, int64_t pool_stride, float cap,
    const bf16_t* __restrict__ talk, const bf16_t* __restrict__ gate, int64_t gate_stride, int n_tokens, float* __restrict__ scores,
    int score_stride) {
    constexpr bool STATS = MODE == 1, KEYS = MODE != 2;
    constexpr int GK = two_pass_gk(HW), HT = GK / 16, NV = 2 * DT, CT = 2 * DT, KPW = BN / TW;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, g4 = lane >> 4;
    bf16_t* Vs = (bf16_t*)(smem + w * NV * 1024);                    // this wave's value tile: rows of dim, 16-byte pieces swizzled
    _Float16* Ps = (_Float16*)(smem + TW * NV * 1024);               // [BN][TT][GK]
    bf16_t* Ms = (bf16_t*)(Ps + BN * TT * GK);                       // [GK][TT][BN]

    const int R = 2 * dim, per = H / G;
    // workgroups go round the XCDs: neighbouring tiles (one sequence's) on one XCD, whose L2 then holds that sequence's rows; the last tile
    // of a run (the most keys) first
    const int per_xcd = gridDim.x / 8, in_order = (int)blockIdx.x < 8 * per_xcd ? (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3) : blockIdx.x;
    const int32_t* tl = tiles + 3 * (gridDim.x - 1 - in_order);
    const int slot = tl[0], t0 = tl[1], ntok = tl[2];
    const int32_t* bt = block_table + (size_t)slot * table_stride;
    const bool row_ok = col < ntok;
    const int t = t0 + (row_ok ? col : 0);
    const int p_row = pos[t], p_first = pos[t0], p_last = pos[t0 + ntok - 1];
    const int lo_row = window > 0 ? max(0, p_row - window + 1) : 0;
    const int kstart = (window > 0 ? max(0, p_first - window + 1) : 0) / BN * BN;
    const int lo_last = window > 0 ? max(0, p_last - window + 1) : 0;
    const int nT = (p_last - kstart) / BN + 1;
    const int Z = gridDim.y, z = blockIdx.y;
    int kv[HW];                                          // key / value pools of the wave's heads (uniform)
#pragma unroll
    for (int i = 0; i < HW; ++i) kv[i] = min(w * HW + i, H - 1) / per;

    v4u q[KEYS ? HW : 1][DT];
#pragma unroll
    for (int i = 0; i < (KEYS ? HW : 0); ++i) {
        const int h = w * HW + i;
        const float* qrow = qf + ((size_t)t * H + min(h, H - 1)) * (size_t)dim;
#pragma unroll
        for (int s = 0; s < DT; ++s) {
            const int e0 = 32 * s + 8 * g4;
            float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
            if (row_ok && h < H && e0 < dim) {
                a = *(const float4*)(qrow + e0);
                b = *(const float4*)(qrow + e0 + 4);
            }
            q[i][s] = v4u{pack_bf2(a.x, a.y), pack_bf2(a.z, a.w), pack_bf2(b.x, b.y), pack_bf2(b.z, b.w)};
        }
    }
    const bool fixed = cap > 0.f && cap <= FIXED_CAP;
    const float c_in = cap > 0.f ? 2.0f * LOG2E / cap : 0.f, c_two = 2.0f * LOG2E * cap;
    float m[HW], l[HW];                                  // STATS: running maximum and sum of this lane's keys; else: m = what comes off
#pragma unroll
    for (int i = 0; i < HW; ++i) {
        l[i] = 0.f;
        m[i] = fixed ? LOG2E * cap : -INFINITY;          // (maxima in units of log 2)
        if (!STATS) {                                    // 2^(score - m) with m = maximum + log2(sum) - 10
            const int h = min(w * HW + i, H - 1);
            float M = -INFINITY, L = 0.f;
            for (int zz = 0; zz < Z1; ++zz) M = fmaxf(M, part_ml[(((size_t)zz * n_tokens + t) * H + h) * 2]);
            for (int zz = 0; zz < Z1; ++zz) {
                const float* ml = part_ml + (((size_t)zz * n_tokens + t) * H + h) * 2;
                L += __builtin_amdgcn_exp2f(ml[0] - M) * ml[1];
            }
            m[i] = M + __builtin_amdgcn_logf(L) - 10.0f;
        }
    }
    v4f acc[STATS ? 1 : HW][STATS ? 1 : CT];
    v4u tf[HT];                                          // talk as A operand: row h = 16 ht + col, columns 8 g4 .. (GK 32) or 4 g4 .. (GK 16)
    const int pieces = dim / 8, inv_pieces = 65536 / pieces + 1;     // (p / pieces = p inv_pieces >> 16 for p < 512, pieces <= 16)
    // 16-byte pieces of a row; piece c of row r lies at c ^ swizzle(r)
    auto swizzle = [&](int row) { return pieces == 16 ? (row & 7) << 1 : pieces == 8 ? ((row >> 1) & 3) << 1 : 0; };
    if (!STATS) {
#pragma unroll
        for (int i = 0; i < HW; ++i)
#pragma unroll
            for (int c = 0; c < CT; ++c) acc[i][c] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) {
            const int h = 16 * ht + col;
            unsigned u[4] = {0u, 0u, 0u, 0u};
#pragma unroll
            for (int e = 0; e < GK / 4; ++e) {
                const int g = GK / 4 * g4 + e;
                const _Float16 v = (_Float16)(h < H && g < H ? bf2f(talk[h * H + g]) : 0.f);
                u[e / 2] |= (unsigned)__builtin_bit_cast(unsigned short, v) << (16 * (e & 1));
            }
            tf[ht] = v4u{u[0], u[1], u[2], u[3]};
        }
        if (TW * HW < GK)                                // heads that no wave owns: zero weights
            for (int i = tid; i < BN * TT * (GK - TW * HW); i += 64 * TW) {
                const int n = GK - TW * HW;
                Ps[(i / n) * GK + TW * HW + i % n] = (_Float16)0.f;
            }
    }
    v4u kr[DT];
    auto tile_base = [&](int tile) {                     // 32 consecutive positions inside one page
        const int k0 = kstart + tile * BN;
        return pool + ((size_t)bt[k0 / page] * page + (size_t)(k0 % page)) * (size_t)R;
    };
    const int k_lane = col * R + dim + 8 * g4;
    auto load_k = [&](const bf16_t* base, int g, int mt) {   // (rows past the last position exist in the page: their weights become zero)
        const bf16_t* b = base + (size_t)g * (size_t)pool_stride + 16 * mt * R + k_lane;
#pragma unroll
        for (int s = 0; s < DT; ++s) kr[s] = 32 * s + 8 * g4 < dim ? *(const v4u*)(b + 32 * s) : v4u{0u, 0u, 0u, 0u};
    };
    auto copy_v = [&](const bf16_t* base, int g, int left) {  // (rows past the last position: the last one again, weight zero)
        const bf16_t* b = base + (size_t)g * (size_t)pool_stride;
        int ln = lane;
        asm volatile("" : "+v"(ln));                     // (addresses made anew per tile: kept across tiles they would cost 16 registers)
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            if (16 * i >= dim) continue;                 // (uniform)
            const int p = ln + 64 * i, r = p * inv_pieces >> 16, row = min(r, BN - 1), c = (p - r * pieces) ^ swizzle(row);
            __builtin_amdgcn_global_load_lds((gptr_t)(b + min(row, left) * R + c * 8), (lptr_t)((unsigned char*)Vs + i * 1024), 16, 0, 0);
        }
    };
    const bf16_t* base = pool;
    if (z < nT) {
        base = tile_base(z);
        if (KEYS) load_k(base, kv[0], 0);
    }
    for (int tile = z; tile < nT; tile += Z) {
        const int k0 = kstart + tile * BN;
        const bf16_t* next = tile + Z < nT ? tile_base(tile + Z) : nullptr;
        if (!STATS) copy_v(base, kv[0], p_last - k0);
        const bool whole = k0 + BN - 1 <= p_first && k0 >= lo_last;      // every token sees every key of the tile
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
            v4f sc[HW];
#pragma unroll
            for (int i = 0; i < HW; ++i) {
                if (!KEYS) {
                    sc[i] = *(const v4f*)(scores + ((size_t)t * H + min(w * HW + i, H - 1)) * (size_t)score_stride + k0 + 16 * mt + 4 * g4);
                    continue;
                }
                if (i > 0 && kv[i] != kv[i > 0 ? i - 1 : 0]) load_k(base, kv[i], mt);
                sc[i] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < DT; ++s)
                    sc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf8, kr[s]), __builtin_bit_cast(bf8, q[KEYS ? i : 0][s]), sc[i], 0, 0, 0);
            }
            if (KEYS) {
                if (mt == 0) load_k(base, kv[0], 1);
                else if (next) load_k(next, kv[0], 0);
            }
            if (HW > 2) __builtin_amdgcn_sched_barrier(0);
            const int key0 = k0 + 16 * mt + 4 * g4;
            unsigned pk[4][HW > 1 ? HW / 2 : 1];         // four keys' weights of this lane's token: the wave's heads in pairs
#pragma unroll
            for (int i = 0; i < HW; ++i) {
                float top = m[i];
#pragma unroll
                for (int r = 0; r < 4; ++r) {            // scores in units of log 2: cap tanh(s / cap) = cap - 2 cap / (2^(c_in s) + 1)
                    if (!KEYS) continue;
                    float x = sc[i][r];
                    if (cap > 0.f) x = LOG2E * cap - c_two * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(c_in * x) + 1.0f);
                    else x *= LOG2E;
                    if (!whole && !(key0 + r <= p_row && key0 + r >= lo_row)) x = -INFINITY;
                    sc[i][r] = x;
                    if (STATS && !fixed) top = fmaxf(top, x);
                }
                if (STATS && scores && row_ok && w * HW + i < H)         // (uniform but for the row)
                    *(v4f*)(scores + ((size_t)t * H + w * HW + i) * (size_t)score_stride + key0) = sc[i];
                if (STATS && !fixed && top > m[i]) {
                    l[i] *= __builtin_amdgcn_exp2f(m[i] - top);          // (first keys: 0 * 2^-inf)
                    m[i] = top;
                }
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float pr = STATS && top == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(sc[i][r] - m[i]);
                    if (STATS) {
                        l[i] += pr;
                    } else {
                        const unsigned u = __builtin_bit_cast(unsigned short, (_Float16)(w * HW + i < H ? pr : 0.f));
                        if (i & 1) pk[r][i / 2] |= u << 16;
                        else pk[r][i / 2] = u;
                    }
                }
                if (HW > 2) __builtin_amdgcn_sched_barrier(0);
            }
            if (!STATS) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    _Float16* dst = Ps + ((16 * mt + 4 * g4 + r) * TT + col) * GK + w * HW;
                    if (HW == 4) *(v2u*)dst = v2u{pk[r][0], pk[r][HW > 2 ? 1 : 0]};
                    else if (HW == 2) *(unsigned*)dst = pk[r][0];
                    else *(unsigned short*)dst = (unsigned short)pk[r][0];
                }
            }
        }
        if (STATS) {
            base = next;
            continue;
        }
        __syncthreads();
        // ---- mix: keys w KPW .. + KPW - 1 of the tile ----
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) {
            v4f mx[KPW];
#pragma unroll
            for (int j = 0; j < KPW; ++j) {
                const _Float16* src = Ps + ((w * KPW + j) * TT + col) * GK + GK / 4 * g4;
                const v4f zero = {0.f, 0.f, 0.f, 0.f};
                if (GK == 32) {
                    mx[j] = __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(h8, tf[ht]), *(const h8*)src, zero, 0, 0, 0);
                } else {
                    const v2u a = {tf[ht][0], tf[ht][1]};
                    mx[j] = __builtin_amdgcn_mfma_f32_16x16x16f16(__builtin_bit_cast(h4, a), *(const h4*)src, zero, 0, 0, 0);
                }
            }
#pragma unroll
            for (int r = 0; r < 4; ++r)
                *(v2u*)(Ms + ((16 * ht + 4 * g4 + r) * TT + col) * BN + w * KPW) =
                    v2u{pack_bf2(mx[0][r], mx[1][r]), pack_bf2(mx[2][r], mx[3][r])};
            if (HT > 1) __builtin_amdgcn_sched_barrier(0);               // (registers: one 16-head block at a time)
        }
        __syncthreads();
        // ---- values: k-slot (g4, e) <-> key 16 (e / 4) + 4 g4 + e % 4 ----
        auto weights = [&](int i) {
            const bf16_t* src = Ms + ((w * HW + i) * TT + col) * BN + 4 * g4;
            const v2u a = *(const v2u*)src, b = *(const v2u*)(src + 16);
            return __builtin_bit_cast(bf8, (v4u{a[0], a[1], b[0], b[1]}));
        };
        const int vr = 4 * g4 + (col >> 2), vsw = swizzle(vr);           // (rows vr and vr + 16 share a swizzle)
        const bf16_t* vrow = Vs + vr * dim + ((col >> 1) & 1) * 8 + (col & 1) * 4;
        auto values = [&](int c) {
            const bf16_t* a = vrow + ((2 * c) ^ vsw) * 8;
            const s4 a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)a);
            const s4 a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4)(a + 16 * dim));
            const v2u u0 = __builtin_bit_cast(v2u, a0), u1 = __builtin_bit_cast(v2u, a1);
            return __builtin_bit_cast(bf8, (v4u{u0[0], u0[1], u1[0], u1[1]}));
        };
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");                 // the value tile has landed (only this wave reads it)
        constexpr int STEP = HW > 1 ? 2 : 1;             // two heads of one pool share a value fragment
#pragma unroll
        for (int i = 0; i < HW; i += STEP) {
            const bool both = STEP == 2 && kv[i] == kv[i + STEP - 1];
#pragma unroll
            for (int half = 0; half < STEP; ++half) {
                const int ii = i + half;
                if (half == 1 && both) continue;         // (done with its neighbour)
                if (ii > 0 && kv[ii] != kv[ii > 0 ? ii - 1 : 0]) {       // (uniform) another pool's values
                    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
                    copy_v(base, kv[ii], p_last - k0);
                    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
                }
                const bf8 p0 = weights(ii), p1 = weights(both ? i + STEP - 1 : ii);
#pragma unroll
                for (int c = 0; c < CT; ++c) {
                    if (16 * c >= dim) continue;         // (uniform)
                    const bf8 a = values(c);
                    acc[ii][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, p0, acc[ii][c], 0, 0, 0);
                    if (STEP == 2 && half == 0 && both)
                        acc[i + STEP - 1][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, p1, acc[i + STEP - 1][c], 0, 0, 0);
                    if (HW > 2 && (c & 1) == 1) __builtin_amdgcn_sched_barrier(0);      // (registers: four fragments ahead at most)
                }
            }
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");               // the value tile has been read: the next copy may start
        base = next;
    }
    if (STATS) {
#pragma unroll
        for (int i = 0; i < HW; ++i) {
            float M = m[i];
            if (!fixed) {
                M = fmaxf(M, __shfl_xor(M, 16, 64));
                M = fmaxf(M, __shfl_xor(M, 32, 64));
                l[i] = M == -INFINITY ? 0.f : l[i] * __builtin_amdgcn_exp2f(m[i] - M);
            }
            float L = l[i];
            L += __shfl_xor(L, 16, 64);
            L += __shfl_xor(L, 32, 64);
            const int h = w * HW + i;
            if (row_ok && h < H && g4 == 0) {
                float* ml = part_ml + (((size_t)z * n_tokens + t) * H + h) * 2;
                ml[0] = M;
                ml[1] = L;
            }
        }
        return;
    }
    if (!row_ok) return;
#pragma unroll
    for (int i = 0; i < HW; ++i) {
        const int h = w * HW + i;
        if (h >= H) continue;
        const float f = 0.0009765625f * (Z == 1 && gate ? 1.0f / (1.0f + __expf(-bf2f(gate[(size_t)t * gate_stride + h]))) : 1.0f);
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const int c0 = 16 * c + 4 * g4;
            if (c0 >= dim) continue;                     // dim % 8 == 0: four values are inside or outside as a whole
            const v4f o = acc[i][c] * f;
            if (Z == 1) *(v2u*)(out + ((size_t)t * H + h) * (size_t)dim + c0) = v2u{pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3])};
            else *(v4f*)(part_o + (((size_t)z * n_tokens + t) * H + h) * (size_t)dim + c0) = o;
        }
    }
}

// out[t, h] = sigmoid(gate[t, h]) sum_z part_o[z, t, h]      (four elements per thread)
__global__ __launch_bounds__(NT) void talking_sum_kernel(bf16_t* __restrict__ out, const float* __restrict__ part_o, const bf16_t* __restrict__ gate,
                                                         int64_t gate_stride, int Z, int H, int dim, int64_t n) {
    const int64_t i = ((int64_t)blockIdx.x * NT + threadIdx.x) * 4;
    if (i >= n) return;
    v4f a = *(const v4f*)(part_o + i);
    for (int z = 1; z < Z; ++z) a += *(const v4f*)(part_o + (int64_t)z * n + i);
    if (gate) {
        const int64_t th = i / dim, t = th / H;
        a *= 1.0f / (1.0f + __expf(-bf2f(gate[t * gate_stride + (th - t * H)])));
    }
    *(v2u*)(out + i) = v2u{pack_bf2(a[0], a[1]), pack_bf2(a[2], a[3])};
}

int pow2_heads(int n) {
    int hp = 1;
    while (hp < n && hp < 16) hp <<= 1;
    return hp;
}
template <typename T>
int launch_wave(float* part_o, const float* qf, const void* pool, const int32_t* bt, int ts, const int32_t* seq, const int32_t* pos, int window,
                int n, int H, int G, int dim, int vdim, int page, int64_t pool_stride, float cap, hipStream_t st_) {
    const dim3 grid(n * H, G), block(NT);
    const int w = dim > vdim ? dim : vdim;
#define QSV_TW(E)                                                                                                              \
    hipLaunchKernelGGL((talking_wave_kernel<T, E>), grid, block, 0, st_, part_o, qf, (const T*)pool, bt, ts, seq, pos, window, H, G, \
                       dim, vdim, page, pool_stride, cap)
    if (w <= 64) QSV_TW(1);
    else if (w <= 128) QSV_TW(2);
    else if (w <= 256) QSV_TW(4);
    else if (w <= 512) QSV_TW(8);
    else {
        qsv_set_error("qsv_talking_attention: heads of %d elements (at most 512)", w);
        return QSV_EINVAL;
    }
#undef QSV_TW
    return QSV_OK;
}
}  // namespace

// Key pools whose heads share a workgroup's rows: prompt tiles 1; steps of few tokens per sequence as many as fill 16 rows and fit 512
// contracted elements.
extern "C" int qsv_talking_attention_key_pools(int heads, int kv_heads, int dim, int decode) {
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0) return 0;
    int kp = 1;
    if (decode)
        for (int c = 2; c <= kv_heads; ++c)
            if (kv_heads % c == 0 && c * (heads / kv_heads) <= 16 && c * dim <= 512) kp = c;
    return kp;
}
extern "C" int qsv_talking_attention_tile_tokens(int heads, int kv_heads, int key_pools) {
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || key_pools <= 0) return 0;
    return NW * (16 / pow2_heads(heads / kv_heads * key_pools));
}
extern "C" int qsv_talking_attention_mfma_ok(int dim, int vdim, int page, int dtype) {
    return dtype == QSV_BF16 && dim % 8 == 0 && vdim % 8 == 0 && dim <= 512 && vdim <= 512 && dim > 0 && vdim > 0 && page % BN == 0;
}

extern "C" int qsv_talking_attention(float* part_o, const float* qf, const void* pool, const int32_t* block_table, int table_stride,
                                     const int32_t* seq, const int32_t* pos, int window, int n, int heads, int kv_heads, int dim, int vdim,
                                     int page, int64_t pool_stride, float cap, int dtype, void* stream) {
    QSV_REQUIRE(part_o && qf && pool && block_table && seq && pos, "qsv_talking_attention: null argument");
    QSV_REQUIRE(n >= 0 && heads > 0 && kv_heads > 0 && kv_heads <= 65535 && heads % kv_heads == 0 && dim > 0 && vdim > 0 && page > 0 && table_stride > 0 &&
                    window >= 0 && pool_stride >= 0 && cap >= 0.f && (int64_t)n * heads < (1ll << 31),
                "qsv_talking_attention: bad sizes (%d heads over %d, %d / %d, page %d)", heads, kv_heads, dim, vdim, page);
    if (n == 0) return QSV_OK;
    int rc = QSV_OK;
    QSV_DISPATCH(dtype, "qsv_talking_attention",
                 rc = launch_wave<T>(part_o, qf, pool, block_table, table_stride, seq, pos, window, n, heads, kv_heads, dim, vdim, page,
                                     pool_stride, cap, (hipStream_t)stream));
    return rc != QSV_OK ? rc : qsv_launch_status("qsv_talking_attention");
}

extern "C" int qsv_talking_attention_mfma(float* part_o, float* part_ml, const float* qf, const void* pool, const int32_t* block_table,
                                          int table_stride, const int32_t* pos, const int32_t* tiles, int n_tiles, int window, int n_tokens,
                                          int heads, int kv_heads, int dim, int vdim, int page, int64_t pool_stride, float cap, int key_pools,
                                          int key_splits, void* stream) {
    QSV_REQUIRE(part_o && part_ml && qf && pool && block_table && pos && tiles, "qsv_talking_attention_mfma: null argument");
    QSV_REQUIRE(qsv_talking_attention_mfma_ok(dim, vdim, page, QSV_BF16) && n_tiles >= 0 && n_tokens >= 0 && table_stride > 0 && window >= 0 &&
                    pool_stride % 8 == 0 && pool_stride >= 0 && cap >= 0.f,
                "qsv_talking_attention_mfma: sizes not supported (dim %d, vdim %d, page %d)", dim, vdim, page);
    QSV_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && key_pools >= 1 && kv_heads % key_pools == 0 && key_pools * dim <= 512 &&
                    key_splits >= 1 && key_splits <= 64,
                "qsv_talking_attention_mfma: %d heads over %d, %d key pools, %d key splits", heads, kv_heads, key_pools, key_splits);
    if (n_tiles == 0) return QSV_OK;
    const int per = heads / kv_heads, rows = per * key_pools, hp = pow2_heads(rows);
    const int ct = (kv_heads * vdim <= 256 || (key_pools == 1 && vdim <= 256)) ? 16 : 32;   // column tiles of a workgroup's values
    int np = 16 * ct / vdim;
    if (np > kv_heads) np = kv_heads;
    const int groups = (kv_heads / key_pools) * ((rows + 15) / 16) * ((kv_heads + np - 1) / np);
    QSV_REQUIRE(groups <= 65535, "qsv_talking_attention_mfma: too many head groups");
    const dim3 grid(n_tiles, groups, key_splits), block(NT);
    const int dt = (key_pools * dim + 31) / 32;
#define QSV_TM(DT, CT)                                                                                                            \
    do {                                                                                                                          \
        size_t lds = (size_t)(BN * k_row(DT) + BN * v_row(np * vdim)) * 2;                                                        \
        const size_t need = (size_t)NW * 64 * (8 * 4 + 2) * 4;           /* merge scratch */                                      \
        if (lds < need) lds = need;                                                                                               \
        if (lds > 64 * 1024) {                                                                                                    \
            const hipError_t e = hipFuncSetAttribute((const void*)talking_mfma_kernel<DT, CT>,                                    \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                       \
            QSV_REQUIRE(e == hipSuccess, "qsv_talking_attention_mfma: %s", hipGetErrorString(e));                                 \
        }                                                                                                                         \
        hipLaunchKernelGGL((talking_mfma_kernel<DT, CT>), grid, block, lds, (hipStream_t)stream, part_o, part_ml, qf,             \
                           (const bf16_t*)pool, block_table, table_stride, pos, tiles, window, heads, kv_heads, dim, vdim, page,  \
                           pool_stride, cap, key_pools, np, hp, 16 / hp, n_tokens);                                               \
    } while (0)
#define QSV_TM_CT(DT)                     \
    do {                                  \
        if (ct == 16) QSV_TM(DT, 16);     \
        else QSV_TM(DT, 32);              \
    } while (0)
    if (dt <= 2) QSV_TM_CT(2);
    else if (dt <= 4) QSV_TM_CT(4);
    else if (dt <= 8) QSV_TM_CT(8);
    else QSV_TM_CT(16);
#undef QSV_TM
#undef QSV_TM_CT
    return qsv_launch_status("qsv_talking_attention_mfma");
}

extern "C" int qsv_talking_mix(void* out, const float* part_o, const float* part_ml, const void* talk, const void* gate, int64_t gate_stride,
                               int key_splits, int n, int heads, int kv_heads, int vdim, int dtype, void* stream) {
    QSV_REQUIRE(out && part_o && talk && n >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && vdim > 0 && key_splits >= 1 &&
                    (part_ml || key_splits == 1) && (!gate || gate_stride >= heads),
                "qsv_talking_mix: bad arguments");
    const size_t lds = ((size_t)key_splits * heads + heads + (size_t)heads * heads) * 4;
    QSV_REQUIRE(lds <= 64 * 1024, "qsv_talking_mix: %d heads in %d key splits do not fit the workgroup's LDS", heads, key_splits);
    if (n == 0) return QSV_OK;
    QSV_DISPATCH(dtype, "qsv_talking_mix",
                 hipLaunchKernelGGL(talking_mix_kernel<T>, dim3(n), dim3(NT), lds, (hipStream_t)stream, (T*)out, part_o, part_ml,
                                    (const T*)talk, (const T*)gate, gate_stride, key_splits, n, heads, kv_heads, vdim));
    return qsv_launch_status("qsv_talking_mix");
}

extern "C" int qsv_talking_two_pass_tile_tokens(void) { return TT; }
extern "C" int qsv_talking_two_pass_ok(int heads, int kv_heads, int dim, int vdim, int page, int dtype) {
    return dtype == QSV_BF16 && heads > 0 && heads <= 32 && kv_heads > 0 && heads % kv_heads == 0 && dim == vdim && dim > 0 && dim % 8 == 0 &&
           dim <= 128 && page % BN == 0;
}
extern "C" int qsv_talking_two_pass(void* out, float* part_o, float* part_ml, const float* qf, const void* pool, const int32_t* block_table,
                                    int table_stride, const int32_t* pos, const int32_t* tiles, int n_tiles, int window, int n_tokens,
                                    int heads, int kv_heads, int dim, int page, int64_t pool_stride, float cap, const void* talk,
                                    const void* gate, int64_t gate_stride, int stat_splits, int key_splits, float* scores, int score_stride,
                                    void* stream) {
    QSV_REQUIRE(out && part_ml && qf && pool && block_table && pos && tiles && talk, "qsv_talking_two_pass: null argument");
    QSV_REQUIRE(qsv_talking_two_pass_ok(heads, kv_heads, dim, dim, page, QSV_BF16) && n_tiles >= 0 && n_tokens >= 0 && table_stride > 0 &&
                    window >= 0 && pool_stride % 8 == 0 && pool_stride >= 0 && cap >= 0.f && (!gate || gate_stride >= heads),
                "qsv_talking_two_pass: sizes not supported (%d heads over %d of %d, page %d)", heads, kv_heads, dim, page);
    QSV_REQUIRE(stat_splits >= 1 && stat_splits <= 64 && key_splits >= 1 && key_splits <= 64 && (key_splits == 1 || part_o),
                "qsv_talking_two_pass: %d / %d key splits", stat_splits, key_splits);
    QSV_REQUIRE(!scores || (score_stride > 0 && score_stride % BN == 0), "qsv_talking_two_pass: score rows of %d keys", score_stride);
    if (n_tiles == 0) return QSV_OK;
    hipStream_t st_ = (hipStream_t)stream;
#define QSV_TP_RUN(HW, DT, MODE, SPLITS, LDS)                                                                                       \
    hipLaunchKernelGGL((talking_two_pass_kernel<HW, DT, MODE>), dim3(n_tiles, SPLITS), dim3(64 * TW), LDS, st_, (bf16_t*)out, part_o, \
                       part_ml, stat_splits, qf, (const bf16_t*)pool, block_table, table_stride, pos, tiles, window, heads, kv_heads, dim, \
                       page, pool_stride, cap, (const bf16_t*)talk, (const bf16_t*)gate, gate_stride, n_tokens, scores, score_stride)
#define QSV_TP_MAIN(HW, DT, MODE)                                                                                                   \
    do {                                                                                                                            \
        const int lds = two_pass_lds(HW, DT);                                                                                       \
        const hipError_t e = hipFuncSetAttribute((const void*)talking_two_pass_kernel<HW, DT, MODE>,                                \
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, lds);                                  \
        QSV_REQUIRE(e == hipSuccess, "qsv_talking_two_pass: %s", hipGetErrorString(e));                                             \
        QSV_TP_RUN(HW, DT, 1, stat_splits, 0);                                                                                      \
        QSV_TP_RUN(HW, DT, MODE, key_splits, lds);                                                                                  \
    } while (0)
#define QSV_TP(HW, DT)                               \
    do {                                             \
        if (scores) QSV_TP_MAIN(HW, DT, 2);          \
        else QSV_TP_MAIN(HW, DT, 0);                 \
    } while (0)
#define QSV_TP_DT(HW)                      \
    do {                                   \
        if (dim <= 64) QSV_TP(HW, 2);      \
        else QSV_TP(HW, 4);                \
    } while (0)
    if (heads <= 8) QSV_TP_DT(1);
    else if (heads <= 16) QSV_TP_DT(2);
    else QSV_TP_DT(4);
#undef QSV_TP
#undef QSV_TP_DT
#undef QSV_TP_MAIN
#undef QSV_TP_RUN
    if (key_splits > 1) {
        const int rc = qsv_launch_status("qsv_talking_two_pass");
        if (rc != QSV_OK) return rc;
        const int64_t n = (int64_t)n_tokens * heads * dim;
        hipLaunchKernelGGL(talking_sum_kernel, dim3((unsigned)((n / 4 + NT - 1) / NT)), dim3(NT), 0, st_, (bf16_t*)out, part_o, (const bf16_t*)gate,
                           gate_stride, key_splits, heads, dim, n);
    }
    return qsv_launch_status("qsv_talking_two_pass");
}
