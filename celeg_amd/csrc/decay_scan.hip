// Linear attention with one decay per head and token, and what lies around it.
//
// Per token and head, with query q and key k (dim numbers, shared by the heads of a group), value v
// (vdim numbers), write strength w and log decay f:
//     S <- exp(f) S + w k v^T;   o = S^T q (+ skip v)
// S [dim, vdim] lives in the request's slot, in 32-bit.  Two kinds:
//  * fixed: f is a number of the head, w = 1; silu may be applied to q, k and v as they are read;
//  * from the input: w = softplus(dt + dt_bias), f = -exp(A_log) w, with dt a column per head.
// Everything behind the projections is 32-bit.
//
// Kernels:
//  * ds_step: one new token of a request (a workgroup per (row, head), one pass over its state);
//  * portions in chunks of 64 rows.  With F_t the sum of f over the chunk's rows up to t,
//        S_t^T q = exp(F_t) S_0^T q + sum_{s <= t} exp(F_t - F_s) w_s (k_s.q) v_s,
//    so nothing in a chunk waits for the token before it:
//      ds_chunk_state: what every chunk adds to the state, and the chunk's whole decay;
//      ds_carry: the states in front of all chunks, and the request's new state;
//      ds_chunk_out: the rows' results.
//    F is summed in double precision and kept as two 32-bit numbers, so that differences keep 32-bit
//    precision however far F runs.  All matrix work runs on the 32-bit matrix instruction (16x16x4).
//  * conv_act: a causal convolution per channel with bias and silu, continuing from the request's saved inputs;
//  * gated_norm: the RMS norm over equal parts of a row with a gate before or behind it.
#include "common.h"

namespace {

typedef float ds_f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 ds_bf16x4 __attribute__((ext_vector_type(4)));

#define DS_ROWS 64        // rows of a chunk
#define DS_THREADS 256

__device__ __forceinline__ float ds_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float ds_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float ds_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// four neighbouring values of a row (vec: they lie on a boundary of four), those from `live` on zero
__device__ __forceinline__ ds_f32x4 ds_load4(const float* p, int live, bool vec) {
    if (vec && live >= 4) return *reinterpret_cast<const ds_f32x4*>(p);
    ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (e < live) v[e] = p[e];
    return v;
}
__device__ __forceinline__ ds_f32x4 ds_load4(const bf16* p, int live, bool vec) {
    ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (vec && live >= 4) {
        const ds_bf16x4 b = *reinterpret_cast<const ds_bf16x4*>(p);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = static_cast<float>(b[e]);
        return v;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (e < live) v[e] = to_float(p[e]);
    return v;
}

struct DsArgs {
    const void *q, *k, *v, *dt;       // rows; group g's query at q + g * D, head h's value at v + h * V, its dt at dt + h
    int ldq, ldk, ldv, ld_dt;
    const float *a_log, *dt_bias;     // with dt
    const float* log_decay;           // without: [H][2], two numbers whose sum is the log
    const float* skip;                // [H] or null
    float* S;
    size_t ldS;                       // distance between slots
    const int *cu_seqlens, *seq_slot, *token_slot;
    float *chunk_s, *chunk_decay;     // [chunk][head][D * V], [chunk][head]
    float* out;
    int ldo;
    int first_seq, n_seqs, n_rows, H, G, D, V, vec, silu;
};

template <typename T>
__device__ __forceinline__ const T* ds_at(const void* base, int row, int ld) {
    return static_cast<const T*>(base) + static_cast<size_t>(row) * ld;
}
__device__ __forceinline__ ds_f32x4 ds_act4(ds_f32x4 x, int silu) {
    if (silu)
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = ds_silu(x[e]);
    return x;
}

// write strength and log decay of (row, head)
template <typename T>
__device__ __forceinline__ void ds_gate(const DsArgs& a, int row, int h, float& w, double& f) {
    if (a.dt) {
        w = ds_softplus(to_float(ds_at<T>(a.dt, row, a.ld_dt)[h]) + a.dt_bias[h]);
        f = static_cast<double>(-expf(a.a_log[h]) * w);
    } else {
        w = 1.f;
        f = static_cast<double>(a.log_decay[2 * h]) + static_cast<double>(a.log_decay[2 * h + 1]);
    }
}

// ---------------------------------------------------------------- one new token
// Threads are laid over (group of rows of S, VEC neighbouring columns).
template <typename T, int VEC>
__global__ __launch_bounds__(DS_THREADS) void ds_step_kernel(const DsArgs a) {
    extern __shared__ float ds_lds[];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, D = a.D, V = a.V;
    const int g0 = h / (a.H / a.G);
    const int n_cols = V / VEC, groups = max(1, DS_THREADS / n_cols);
    float* qs = ds_lds;
    float* ks = qs + D;
    float* vs = ks + D;
    float* part = vs + V;             // [groups][V]
    const size_t slot = static_cast<size_t>(a.token_slot[t]);
    float w;
    double f;
    ds_gate<T>(a, t, h, w, f);
    const float keep = expf(static_cast<float>(f));
    const T* q_row = ds_at<T>(a.q, t, a.ldq) + g0 * D;
    const T* k_row = ds_at<T>(a.k, t, a.ldk) + g0 * D;
    const T* v_row = ds_at<T>(a.v, t, a.ldv) + h * V;
    for (int d = tid; d < D; d += DS_THREADS) {
        const float q = to_float(q_row[d]), k = to_float(k_row[d]);
        qs[d] = a.silu ? ds_silu(q) : q;
        ks[d] = (a.silu ? ds_silu(k) : k) * w;
    }
    for (int j = tid; j < V; j += DS_THREADS) {
        const float v = to_float(v_row[j]);
        vs[j] = a.silu ? ds_silu(v) : v;
    }
    __syncthreads();

    float* S = a.S + slot * a.ldS + static_cast<size_t>(h) * D * V;
    const int g = tid / n_cols;
    if (g < groups) {
        for (int c = tid % n_cols; c < n_cols; c += DS_THREADS) {
            float value[VEC], acc[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                value[e] = vs[c * VEC + e];
                acc[e] = 0.f;
            }
            auto update = [&](int d, float (&s)[VEC]) __attribute__((always_inline)) {
                const float k = ks[d], q = qs[d];
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    s[e] = fmaf(k, value[e], keep * s[e]);
                    acc[e] = fmaf(q, s[e], acc[e]);
                }
            };
            auto fetch = [&](int d, float (&s)[VEC]) __attribute__((always_inline)) {
                const float* p = S + static_cast<size_t>(d) * V + c * VEC;
                if (VEC == 4) {
                    const ds_f32x4 x = *reinterpret_cast<const ds_f32x4*>(p);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) s[e] = x[e];
                } else {
                    s[0] = p[0];
                }
            };
            auto store = [&](int d, const float (&s)[VEC]) __attribute__((always_inline)) {
                float* p = S + static_cast<size_t>(d) * V + c * VEC;
                if (VEC == 4) *reinterpret_cast<ds_f32x4*>(p) = ds_f32x4{s[0], s[VEC > 1 ? 1 : 0], s[VEC > 2 ? 2 : 0], s[VEC > 3 ? 3 : 0]};
                else p[0] = s[0];
            };
            int d = g;
            for (; d + 7 * groups < D; d += 8 * groups) {      // eight rows asked for together
                float s[8][VEC];
#pragma unroll
                for (int u = 0; u < 8; ++u) fetch(d + u * groups, s[u]);
#pragma unroll
                for (int u = 0; u < 8; ++u) update(d + u * groups, s[u]);
#pragma unroll
                for (int u = 0; u < 8; ++u) store(d + u * groups, s[u]);
            }
            for (; d < D; d += groups) {
                float s[VEC];
                fetch(d, s);
                update(d, s);
                store(d, s);
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) part[static_cast<size_t>(g) * V + c * VEC + e] = acc[e];
        }
    }
    __syncthreads();
    const float skip = a.skip ? a.skip[h] : 0.f;
    float* out = a.out + static_cast<size_t>(t) * a.ldo + static_cast<size_t>(h) * V;
    for (int j = tid; j < V; j += DS_THREADS) {
        float o = skip * vs[j];
        for (int u = 0; u < groups; ++u) o += part[static_cast<size_t>(u) * V + j];
        out[j] = o;
    }
}

// ---------------------------------------------------------------- portions
// which request and chunk of it: the chunks of the requests from first_seq on, one after the other
__device__ __forceinline__ bool ds_find_chunk(const DsArgs& a, int index, int& s, int& row0, int& rows) {
    int chunk = index;
    for (s = a.first_seq; s < a.n_seqs; ++s) {
        const int start = a.cu_seqlens[s], n = a.cu_seqlens[s + 1] - start;
        const int chunks = (n + DS_ROWS - 1) / DS_ROWS;
        if (chunk < chunks) {
            row0 = start + chunk * DS_ROWS;
            rows = min(DS_ROWS, n - chunk * DS_ROWS);
            return true;
        }
        chunk -= chunks;
    }
    return false;
}

// The chunk's gates into LDS, by the first wavefront: w [64], F as two numbers [64] each (rows past the
// end: w 0, F as the last row's).  The caller's next barrier ends the writing.
template <typename T>
__device__ __forceinline__ void ds_chunk_gates(const DsArgs& a, int h, int row0, int rows, float* w_s, float* hi_s, float* lo_s) {
    if (threadIdx.x >= CELEG_WAVE) return;
    const int lane = threadIdx.x;
    float w = 0.f;
    double F = 0.0;
    if (lane < rows) ds_gate<T>(a, row0 + lane, h, w, F);
#pragma unroll
    for (int off = 1; off < CELEG_WAVE; off <<= 1) {
        const double y = __shfl_up(F, off, CELEG_WAVE);
        if (lane >= off) F += y;
    }
    const float hi = static_cast<float>(F);
    w_s[lane] = w;
    hi_s[lane] = hi;
    lo_s[lane] = static_cast<float>(F - static_cast<double>(hi));
}

// What a chunk adds to the state: one workgroup per (chunk, head, 64 columns).
template <typename T>
__global__ __launch_bounds__(256) void ds_chunk_state_kernel(const DsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float ds_lds[];
    __shared__ float w_s[DS_ROWS], hi_s[DS_ROWS], lo_s[DS_ROWS];
    const int D = a.D, V = a.V, Dp = (D + 15) & ~15, KROW = Dp + 4, VROW = 64 + 4;
    float* Ks = ds_lds;                       // [64][KROW], weighted
    float* Vs = Ks + DS_ROWS * KROW;          // [64][VROW]
    int s, row0, rows;
    if (!ds_find_chunk(a, blockIdx.x, s, row0, rows)) return;
    const int h = blockIdx.y, g0 = h / (a.H / a.G), col0 = blockIdx.z * 64;
    const int tid = threadIdx.x, lane = tid % CELEG_WAVE, wave = tid / CELEG_WAVE, c = lane & 15, quad = lane >> 4;
    ds_chunk_gates<T>(a, h, row0, rows, w_s, hi_s, lo_s);
    __syncthreads();
    const float last_hi = hi_s[rows - 1], last_lo = lo_s[rows - 1];
    for (int i = tid; i < DS_ROWS * (Dp / 4); i += 256) {
        const int r = i / (Dp / 4), d = 4 * (i % (Dp / 4));
        ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows && d < D) {
            const float w = w_s[r] * expf((last_hi - hi_s[r]) + (last_lo - lo_s[r]));
            v = ds_act4(ds_load4(ds_at<T>(a.k, row0 + r, a.ldk) + g0 * D + d, D - d, a.vec), a.silu) * w;
        }
        *reinterpret_cast<ds_f32x4*>(Ks + r * KROW + d) = v;
    }
    for (int i = tid; i < DS_ROWS * 16; i += 256) {
        const int r = i / 16, j = 4 * (i % 16);
        ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows && col0 + j < V) v = ds_act4(ds_load4(ds_at<T>(a.v, row0 + r, a.ldv) + h * V + col0 + j, V - col0 - j, a.vec), a.silu);
        *reinterpret_cast<ds_f32x4*>(Vs + r * VROW + j) = v;
    }
    __syncthreads();
    const size_t at = static_cast<size_t>(blockIdx.x) * a.H + h;
    if (blockIdx.z == 0 && tid == 0) a.chunk_decay[at] = expf(last_hi + last_lo);
    float* out = a.chunk_s + at * D * V;
    const int groups = (rows + 15) / 16;
    for (int dt = wave; dt < Dp / 16; dt += 4) {
        ds_f32x4 acc[4];
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) acc[ct] = ds_f32x4{0.f, 0.f, 0.f, 0.f};
        for (int g = 0; g < groups; ++g)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int r = 16 * g + 4 * quad + e;
                const float k = Ks[r * KROW + 16 * dt + c];
#pragma unroll
                for (int ct = 0; ct < 4; ++ct) acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, Vs[r * VROW + 16 * ct + c], acc[ct], 0, 0, 0);
            }
#pragma unroll
        for (int ct = 0; ct < 4; ++ct)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * dt + 4 * quad + i, j = col0 + 16 * ct + c;
                if (d < D && j < V) out[static_cast<size_t>(d) * V + j] = acc[ct][i];
            }
    }
}

// The states in front of the chunks: a thread per number of S and (request, head); chunk by chunk, what
// the chunk adds makes room for the state in front of it; what is left at the end is the new state.
__global__ __launch_bounds__(256) void ds_carry_kernel(const DsArgs a) {
    const int e = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, s = a.first_seq + blockIdx.z;
    const int per_s = a.D * a.V;
    if (e >= per_s) return;
    int chunk0 = 0;
    for (int p = a.first_seq; p < s; ++p) chunk0 += (a.cu_seqlens[p + 1] - a.cu_seqlens[p] + DS_ROWS - 1) / DS_ROWS;
    const int n = a.cu_seqlens[s + 1] - a.cu_seqlens[s];
    if (n <= 0) return;
    float* mine = a.S + static_cast<size_t>(a.seq_slot[s]) * a.ldS + static_cast<size_t>(h) * per_s + e;
    const size_t step = static_cast<size_t>(a.H) * per_s;
    float* at = a.chunk_s + (static_cast<size_t>(chunk0) * a.H + h) * per_s + e;
    const float* decay = a.chunk_decay + static_cast<size_t>(chunk0) * a.H + h;
    float x = *mine;
    const int chunks = (n + DS_ROWS - 1) / DS_ROWS;
    int i = 0;
    for (; i + 8 <= chunks; i += 8) {
        float added[8], keep[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            added[u] = at[(i + u) * step];
            keep[u] = decay[static_cast<size_t>(i + u) * a.H];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            at[(i + u) * step] = x;
            x = fmaf(keep[u], x, added[u]);
        }
    }
    for (; i < chunks; ++i) {
        const float added = at[i * step];
        at[i * step] = x;
        x = fmaf(decay[static_cast<size_t>(i) * a.H], x, added);
    }
    *mine = x;
}

// The rows' results: one workgroup of four wavefronts per (chunk, head), 16 rows a wavefront.  KG: groups
// of 16 key numbers (an upper bound of the head's).
template <typename T, int KG>
__global__ __launch_bounds__(256) void ds_chunk_out_kernel(const DsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float ds_lds[];
    __shared__ float w_s[DS_ROWS], hi_s[DS_ROWS], lo_s[DS_ROWS];
    const int D = a.D, V = a.V, Dp = (D + 15) & ~15, KROW = Dp + 4;
    constexpr int PROW = DS_ROWS + 4, VROW = 64 + 4;
    float* Vs = ds_lds;                              // [64][VROW]
    float* Ks = Vs + DS_ROWS * VROW;                 // [64][KROW]; later the rows' weights, [4][16][PROW]
    int s, row0, rows;
    if (!ds_find_chunk(a, blockIdx.x, s, row0, rows)) return;
    const int h = blockIdx.y, g0 = h / (a.H / a.G);
    const int tid = threadIdx.x, lane = tid % CELEG_WAVE, wave = tid / CELEG_WAVE, c = lane & 15, quad = lane >> 4;
    const float* S0 = a.chunk_s + (static_cast<size_t>(blockIdx.x) * a.H + h) * D * V;
    const bool vec = a.vec != 0;

    // this wavefront's queries: lane (c, quad) holds numbers 16 g + 4 quad .. + 3 of row 16 wave + c
    const int q_row = 16 * wave + c;
    ds_f32x4 q[KG];
#pragma unroll
    for (int g = 0; g < KG; ++g) {
        const int d = 16 * g + 4 * quad;
        q[g] = ds_f32x4{0.f, 0.f, 0.f, 0.f};
        if (d < D && q_row < rows) q[g] = ds_act4(ds_load4(ds_at<T>(a.q, row0 + q_row, a.ldq) + g0 * D + d, D - d, vec), a.silu);
    }
    ds_chunk_gates<T>(a, h, row0, rows, w_s, hi_s, lo_s);
    for (int i = tid; i < DS_ROWS * (Dp / 4); i += 256) {
        const int r = i / (Dp / 4), d = 4 * (i % (Dp / 4));
        ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows && d < D) v = ds_act4(ds_load4(ds_at<T>(a.k, row0 + r, a.ldk) + g0 * D + d, D - d, vec), a.silu);
        *reinterpret_cast<ds_f32x4*>(Ks + r * KROW + d) = v;
    }
    __syncthreads();

    // the numbers of this lane's result rows, 16 wave + 4 quad + i
    float f_hi[4], f_lo[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        f_hi[i] = hi_s[16 * wave + 4 * quad + i];
        f_lo[i] = lo_s[16 * wave + 4 * quad + i];
    }
    ds_f32x4 weight[4];                               // of this lane's rows, for key 16 st + c
#pragma unroll
    for (int st = 0; st < 4; ++st) {
        weight[st] = ds_f32x4{0.f, 0.f, 0.f, 0.f};
        if (st > wave) continue;                      // keys behind the wavefront's last row are not seen
        ds_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int g = 0; g < KG; ++g)
            if (16 * g < D) {
                const ds_f32x4 k = *reinterpret_cast<const ds_f32x4*>(Ks + (16 * st + c) * KROW + 16 * g + 4 * quad);
#pragma unroll
                for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q[g][e], k[e], acc, 0, 0, 0);
            }
        const int key = 16 * st + c;
        const float in_hi = hi_s[key], in_lo = lo_s[key], w = w_s[key];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * quad + i;
            weight[st][i] = key <= t ? acc[i] * w * expf((f_hi[i] - in_hi) + (f_lo[i] - in_lo)) : 0.f;
        }
    }
    __syncthreads();                                  // (the keys have been read; the weights take their place)
    float* mine = Ks + wave * 16 * PROW;
#pragma unroll
    for (int st = 0; st < 4; ++st)
        if (st <= wave)
#pragma unroll
            for (int i = 0; i < 4; ++i) mine[(4 * quad + i) * PROW + 16 * st + c] = weight[st][i];
    float carry[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) carry[i] = expf(f_hi[i] + f_lo[i]);
    const float skip = a.skip ? a.skip[h] : 0.f;
    for (int ct = 0; ct < (V + 15) / 16; ++ct) {
        if (ct % 4 == 0) {
            __syncthreads();
            for (int i = tid; i < DS_ROWS * 16; i += 256) {
                const int r = i / 16, j = 16 * ct + 4 * (i % 16);
                ds_f32x4 v = {0.f, 0.f, 0.f, 0.f};
                if (r < rows && j < V) v = ds_act4(ds_load4(ds_at<T>(a.v, row0 + r, a.ldv) + h * V + j, V - j, vec), a.silu);
                *reinterpret_cast<ds_f32x4*>(Vs + r * VROW + 4 * (i % 16)) = v;
            }
            __syncthreads();
        }
        const int j = 16 * ct + c;
        const bool has = j < V;
        ds_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int g = 0; g < KG; ++g)
            if (16 * g < D) {
                float b[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int d = 16 * g + 4 * quad + e;
                    b[e] = has && d < D ? S0[static_cast<size_t>(d) * V + j] : 0.f;
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q[g][e], b[e], acc, 0, 0, 0);
            }
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] *= carry[i];
        for (int g = 0; g <= wave; ++g) {
            const ds_f32x4 p = *reinterpret_cast<const ds_f32x4*>(mine + c * PROW + 16 * g + 4 * quad);
#pragma unroll
            for (int e = 0; e < 4; ++e)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(p[e], Vs[(16 * g + 4 * quad + e) * VROW + 16 * (ct % 4) + c], acc, 0, 0, 0);
        }
        if (has)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * wave + 4 * quad + i;
                if (t >= rows) continue;
                a.out[static_cast<size_t>(row0 + t) * a.ldo + static_cast<size_t>(h) * V + j] =
                    fmaf(skip, Vs[t * VROW + 16 * (ct % 4) + c], acc[i]);
            }
    }
}

int ds_allow(const void* kernel, size_t lds) {
    if (lds <= 64 * 1024) return 0;
    return static_cast<int>(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)));
}

template <typename T, int KG>
int ds_out_launch(const DsArgs& a, int max_chunks, size_t lds, hipStream_t stream) {
    auto kernel = ds_chunk_out_kernel<T, KG>;
    if (int rc = ds_allow(reinterpret_cast<const void*>(kernel), lds)) return rc;
    hipLaunchKernelGGL(kernel, dim3(max_chunks, a.H), dim3(256), lds, stream, a);
    return CELEG_LAUNCH_RESULT();
}

template <typename T>
int ds_rows(const DsArgs& a, int max_chunks, hipStream_t stream) {
    const int Dp = (a.D + 15) & ~15, seqs = a.n_seqs - a.first_seq;
    const size_t state_lds = (static_cast<size_t>(DS_ROWS) * (Dp + 4) + DS_ROWS * 68) * sizeof(float);
    if (int rc = ds_allow(reinterpret_cast<const void*>(ds_chunk_state_kernel<T>), state_lds)) return rc;
    hipLaunchKernelGGL(ds_chunk_state_kernel<T>, dim3(max_chunks, a.H, (a.V + 63) / 64), dim3(256), state_lds, stream, a);
    if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    hipLaunchKernelGGL(ds_carry_kernel, dim3((a.D * a.V + 255) / 256, a.H, seqs), dim3(256), 0, stream, a);
    if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    const size_t k_floats = static_cast<size_t>(DS_ROWS) * (Dp + 4), p_floats = 4 * 16 * (DS_ROWS + 4);
    const size_t out_lds = (DS_ROWS * 68 + (k_floats > p_floats ? k_floats : p_floats)) * sizeof(float);
    if (Dp <= 64) return ds_out_launch<T, 4>(a, max_chunks, out_lds, stream);
    if (Dp <= 128) return ds_out_launch<T, 8>(a, max_chunks, out_lds, stream);
    return ds_out_launch<T, 16>(a, max_chunks, out_lds, stream);
}

// ---------------------------------------------------------------- convolution with bias and silu
// y_t[c] = silu(bias[c] + sum_j w[j, c] u_(t - taps + 1 + j)[c]); saved [slots][taps - 1][channels] keeps a
// request's last inputs.  A thread owns VEC neighbouring channels of rows_each rows.  The first taps - 1 rows of
// a portion, the only ones that read the saved inputs, are all computed by the block that holds the portion's
// first row, whose threads then leave the new inputs.
// TAPS: their number where it is known to the compiler (the inputs then move through registers), 0: any.
// (also gated_norm's loads)
template <typename T, int VEC>
__device__ __forceinline__ void conv_load(const T* p, float (&x)[VEC]) {
    if (VEC == 4) {
        const ds_f32x4 v = ds_load4(p, 4, true);
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[e] = v[e];
    } else {
        x[0] = to_float(p[0]);
    }
}
template <typename T, int VEC>
__device__ __forceinline__ void conv_store(T* p, const float (&y)[VEC]) {
    float z[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) z[e] = ds_silu(y[e]);
    if constexpr (VEC == 4) Vec4<T>::store(p, z);
    else p[0] = from_float<T>(z[0]);
}

template <typename T, int VEC, int TAPS>
__global__ __launch_bounds__(CELEG_WAVE) void conv_act_kernel(const T* __restrict__ u, int ldu, const float* __restrict__ w,
                                                              const float* __restrict__ bias, float* __restrict__ state,
                                                              size_t state_stride, const int* __restrict__ token_seq,
                                                              const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slot,
                                                              T* __restrict__ out, int ldo, int n_rows, int channels, int n_taps, int rows_each) {
    const int taps = TAPS > 0 ? TAPS : n_taps;
    const int c = (blockIdx.x * CELEG_WAVE + threadIdx.x) * VEC;
    if (c >= channels) return;
    const int r0 = blockIdx.y * rows_each, r1 = min(r0 + rows_each, n_rows);
    const T* mine = u + c;
    float held_w[TAPS > 0 ? TAPS : 1][VEC], b[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) b[e] = bias ? bias[c + e] : 0.f;
    if (TAPS > 0)
#pragma unroll
        for (int j = 0; j < (TAPS > 0 ? TAPS : 1); ++j) conv_load<float, VEC>(w + static_cast<size_t>(j) * channels + c, held_w[j]);
    auto weight = [&](int j, float (&x)[VEC]) __attribute__((always_inline)) { conv_load<float, VEC>(w + static_cast<size_t>(j) * channels + c, x); };
    for (int t = r0; t < r1;) {
        const int s = token_seq[t], first = cu_seqlens[s], end = cu_seqlens[s + 1];
        const int stop = min(end, r1);
        if (first >= r0) {
            float* saved = state + static_cast<size_t>(seq_slot[s]) * state_stride + c;
            const int edge = min(end, first + taps - 1);
            for (int x = first; x < edge; ++x) {
                float y[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[e] = b[e];
                for (int j = 0; j < taps; ++j) {
                    const int from = x - first - (taps - 1 - j);       // place of the input in the portion
                    float v[VEC], wj[VEC];
                    weight(j, wj);
                    if (from >= 0) conv_load<T, VEC>(mine + static_cast<size_t>(first + from) * ldu, v);
                    else conv_load<float, VEC>(saved + static_cast<size_t>(taps - 1 + from) * channels, v);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y[e] = fmaf(wj[e], v[e], y[e]);
                }
                conv_store<T, VEC>(out + static_cast<size_t>(x) * ldo + c, y);
            }
            // (its own block alone reads them, and it has: the inputs that the request's next row will look back to)
            const int n = end - first;
            for (int j = 0; j < taps - 1; ++j) {
                const int from = n - (taps - 1) + j;
                float v[VEC];
                if (from >= 0) conv_load<T, VEC>(mine + static_cast<size_t>(first + from) * ldu, v);
                else conv_load<float, VEC>(saved + static_cast<size_t>(taps - 1 + from) * channels, v);
#pragma unroll
                for (int e = 0; e < VEC; ++e) saved[static_cast<size_t>(j) * channels + e] = v[e];
            }
        }
        const int from = max(t, first + taps - 1);
        if (from < stop) {
            if (TAPS > 1) {
                float in[TAPS > 1 ? TAPS : 1][VEC];
#pragma unroll
                for (int j = 0; j < TAPS - 1; ++j) conv_load<T, VEC>(mine + static_cast<size_t>(from - (TAPS - 1) + j) * ldu, in[j]);
                for (int x = from; x < stop; ++x) {
                    conv_load<T, VEC>(mine + static_cast<size_t>(x) * ldu, in[TAPS > 1 ? TAPS - 1 : 0]);
                    float y[VEC];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) {
                        y[e] = b[e];
#pragma unroll
                        for (int j = 0; j < TAPS; ++j) y[e] = fmaf(held_w[j][e], in[j][e], y[e]);
#pragma unroll
                        for (int j = 0; j < TAPS - 1; ++j) in[j][e] = in[j + 1][e];
                    }
                    conv_store<T, VEC>(out + static_cast<size_t>(x) * ldo + c, y);
                }
            } else {
                for (int x = from; x < stop; ++x) {
                    float y[VEC];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y[e] = b[e];
                    for (int j = 0; j < taps; ++j) {
                        float v[VEC], wj[VEC];
                        weight(j, wj);
                        conv_load<T, VEC>(mine + static_cast<size_t>(x - (taps - 1 - j)) * ldu, v);
#pragma unroll
                        for (int e = 0; e < VEC; ++e) y[e] = fmaf(wj[e], v[e], y[e]);
                    }
                    conv_store<T, VEC>(out + static_cast<size_t>(x) * ldo + c, y);
                }
            }
        }
        t = stop;
    }
}

// ---------------------------------------------------------------- gate and norm
// One workgroup per (row, part).  mode 0: o / rms(o) * weight * sigmoid(gate); mode 1: y = o * silu(gate), then
// y / rms(y) * weight.  The mean of squares runs over the part's `size` values.
// VEC neighbouring values a thread and turn.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gated_norm_kernel(const float* __restrict__ o, int ldo, const T* __restrict__ gate, int ldg,
                                                         const float* __restrict__ weight, T* __restrict__ out, int ld, int size,
                                                         float eps, int mode) {
    __shared__ float scratch[16];
    constexpr int HELD = VEC == 4 ? 4 : 8;
    const size_t t = blockIdx.x;
    const int base = blockIdx.y * size, first = threadIdx.x * VEC, step = blockDim.x * VEC;
    const float* x = o + t * ldo + base;
    const T* g = gate + t * ldg + base;
    const float* w = weight + base;
    auto fetch = [&](int i, float (&y)[VEC], float (&z)[VEC]) __attribute__((always_inline)) {     // values (gated in mode 1) and gates
        conv_load<float, VEC>(x + i, y);
        conv_load<T, VEC>(g + i, z);
        if (mode == 1)
#pragma unroll
            for (int e = 0; e < VEC; ++e) y[e] *= ds_silu(z[e]);
    };
    float held[HELD][VEC], held_z[HELD][VEC], sq = 0.f;
#pragma unroll
    for (int u = 0; u < HELD; ++u) {
        const int i = first + u * step;
        if (i < size) {
            fetch(i, held[u], held_z[u]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) sq = fmaf(held[u][e], held[u][e], sq);
        }
    }
    for (int i = first + HELD * step; i < size; i += step) {
        float y[VEC], z[VEC];
        fetch(i, y, z);
#pragma unroll
        for (int e = 0; e < VEC; ++e) sq = fmaf(y[e], y[e], sq);
    }
    sq = block_sum(sq, scratch);
    const float unit = 1.0f / sqrtf(sq / static_cast<float>(size) + eps);
    T* dst = out + t * ld + base;
    auto finish = [&](int i, float (&y)[VEC], const float (&z)[VEC]) __attribute__((always_inline)) {
        float wv[VEC];
        conv_load<float, VEC>(w + i, wv);
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            y[e] *= unit * wv[e];
            if (mode == 0) y[e] *= ds_sigmoid(z[e]);
        }
        if constexpr (VEC == 4) Vec4<T>::store(dst + i, y);
        else dst[i] = from_float<T>(y[0]);
    };
#pragma unroll
    for (int u = 0; u < HELD; ++u) {
        const int i = first + u * step;
        if (i < size) finish(i, held[u], held_z[u]);
    }
    for (int i = first + HELD * step; i < size; i += step) {
        float y[VEC], z[VEC];
        fetch(i, y, z);
        finish(i, y, z);
    }
}

}  // namespace

// q, k [rows, G * D] and v [rows, H * V] with their row strides; dt (columns per head) with a_log and dt_bias, or null
// with log_decay [H][2].  Rows [0, n_single) are requests of one new token; the requests from n_single on bring portions,
// whose chunks of 64 rows are at most max_chunks.  chunk_s: room for max_chunks * H * D * V numbers, chunk_decay for
// max_chunks * H.
extern "C" int celeg_decay_scan(const void* q, int ldq, const void* k, int ldk, const void* v, int ldv, int dtype, const void* dt,
                                int ld_dt, const float* a_log, const float* dt_bias, const float* log_decay, const float* skip, int silu,
                                float* S, size_t ldS, const int* cu_seqlens, const int* seq_slot, const int* token_slot, float* chunk_s,
                                float* chunk_decay, float* out, int ldo, int n_rows, int n_seqs, int n_single, int max_chunks, int H,
                                int G, int D, int V, hipStream_t stream) {
    if (n_rows <= 0 || n_seqs <= 0) return 0;
    if (H <= 0 || G <= 0 || H % G || D <= 0 || V <= 0 || D > 256 || V > 4096 || n_single < 0 || n_single > n_seqs ||
        (dt ? !a_log || !dt_bias : !log_decay))
        return static_cast<int>(hipErrorInvalidValue);
    DsArgs a;
    a.q = q;
    a.k = k;
    a.v = v;
    a.dt = dt;
    a.ldq = ldq;
    a.ldk = ldk;
    a.ldv = ldv;
    a.ld_dt = ld_dt;
    a.a_log = a_log;
    a.dt_bias = dt_bias;
    a.log_decay = log_decay;
    a.skip = skip;
    a.S = S;
    a.ldS = ldS;
    a.cu_seqlens = cu_seqlens;
    a.seq_slot = seq_slot;
    a.token_slot = token_slot;
    a.chunk_s = chunk_s;
    a.chunk_decay = chunk_decay;
    a.out = out;
    a.ldo = ldo;
    a.first_seq = n_single;
    a.n_seqs = n_seqs;
    a.n_rows = n_rows;
    a.H = H;
    a.G = G;
    a.D = D;
    a.V = V;
    a.silu = silu;
    const uintptr_t four = dtype == CELEG_F32 ? 16 : 8;
    const uintptr_t ends = reinterpret_cast<uintptr_t>(q) | reinterpret_cast<uintptr_t>(k) | reinterpret_cast<uintptr_t>(v);
    a.vec = ((ldq | ldk | ldv | D | V) & 3) == 0 && (ends & (four - 1)) == 0;
    if (n_single > 0) {
        // four columns a thread where the states allow it
        const bool by_fours = V % 4 == 0 && ldS % 4 == 0 && (reinterpret_cast<uintptr_t>(S) & 15) == 0;
        const int n_cols = by_fours ? V / 4 : V, groups = n_cols >= DS_THREADS ? 1 : DS_THREADS / n_cols;
        const size_t lds = (2 * static_cast<size_t>(D) + V + static_cast<size_t>(groups) * V) * sizeof(float);
        dim3 grid(n_single, H), block(DS_THREADS);
        if (dtype == CELEG_F32 && by_fours) hipLaunchKernelGGL((ds_step_kernel<float, 4>), grid, block, lds, stream, a);
        else if (dtype == CELEG_F32) hipLaunchKernelGGL((ds_step_kernel<float, 1>), grid, block, lds, stream, a);
        else if (by_fours) hipLaunchKernelGGL((ds_step_kernel<bf16, 4>), grid, block, lds, stream, a);
        else hipLaunchKernelGGL((ds_step_kernel<bf16, 1>), grid, block, lds, stream, a);
        if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    }
    if (n_seqs == n_single) return 0;
    if (max_chunks <= 0 || !chunk_s || !chunk_decay) return static_cast<int>(hipErrorInvalidValue);
    return dtype == CELEG_F32 ? ds_rows<float>(a, max_chunks, stream) : ds_rows<bf16>(a, max_chunks, stream);
}

extern "C" int celeg_conv_act(const void* u, int ldu, int dtype, const float* w, const float* bias, float* state, size_t state_stride,
                              const int* token_seq, const int* cu_seqlens, const int* seq_slot, void* out, int ldo, int n_rows,
                              int channels, int taps, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (channels <= 0 || taps <= 0) return static_cast<int>(hipErrorInvalidValue);
    const uintptr_t four = dtype == CELEG_F32 ? 16 : 8;
    // (weights and saved inputs are read by fours as well)
    const bool by_fours = ((channels | ldu | ldo) & 3) == 0 && (state_stride & 3) == 0 &&
                          ((reinterpret_cast<uintptr_t>(u) | reinterpret_cast<uintptr_t>(out)) & (four - 1)) == 0 &&
                          ((reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(state)) & 15) == 0;
    const int per_block = CELEG_WAVE * (by_fours ? 4 : 1);
    const int rows_each = n_rows <= 128 ? 1 : 8;         // (few rows: latency is what counts)
    dim3 grid((channels + per_block - 1) / per_block, (n_rows + rows_each - 1) / rows_each), block(CELEG_WAVE);
#define CONV_GO_TAPS(T, VEC, TAPS)                                                                                                   \
    hipLaunchKernelGGL((conv_act_kernel<T, VEC, TAPS>), grid, block, 0, stream, static_cast<const T*>(u), ldu, w, bias, state, state_stride, \
                       token_seq, cu_seqlens, seq_slot, static_cast<T*>(out), ldo, n_rows, channels, taps, rows_each)
#define CONV_GO(T, VEC)                        \
    switch (taps) {                            \
        case 2: CONV_GO_TAPS(T, VEC, 2); break; \
        case 3: CONV_GO_TAPS(T, VEC, 3); break; \
        case 4: CONV_GO_TAPS(T, VEC, 4); break; \
        default: CONV_GO_TAPS(T, VEC, 0);      \
    }
    if (dtype == CELEG_F32 && by_fours) {
        CONV_GO(float, 4)
    } else if (dtype == CELEG_F32) {
        CONV_GO(float, 1)
    } else if (by_fours) {
        CONV_GO(bf16, 4)
    } else {
        CONV_GO(bf16, 1)
    }
#undef CONV_GO
#undef CONV_GO_TAPS
    return CELEG_LAUNCH_RESULT();
}

// o [rows, parts * size] 32-bit, gate rows of the same width
extern "C" int celeg_gated_norm(const float* o, int ldo, const void* gate, int ldg, int dtype, const float* weight, void* out, int ld,
                                int rows, int parts, int size, float eps, int mode, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (parts <= 0 || parts > 65535 || size <= 0 || mode < 0 || mode > 1) return static_cast<int>(hipErrorInvalidValue);
    const uintptr_t ends = reinterpret_cast<uintptr_t>(o) | reinterpret_cast<uintptr_t>(gate) | reinterpret_cast<uintptr_t>(weight) |
                           reinterpret_cast<uintptr_t>(out);
    const uintptr_t half = dtype == CELEG_F32 ? 15 : 7;
    const bool by_fours = ((size | ldo | ldg | ld) & 3) == 0 && (ends & half) == 0 && ((reinterpret_cast<uintptr_t>(o) | reinterpret_cast<uintptr_t>(weight)) & 15) == 0;
    const int turns = by_fours ? size / 4 : size;
    dim3 grid(rows, parts), block(turns <= 64 ? 64 : turns <= 128 ? 128 : 256);
#define NORM_GO(T, VEC)                                                                                                              \
    hipLaunchKernelGGL((gated_norm_kernel<T, VEC>), grid, block, 0, stream, o, ldo, static_cast<const T*>(gate), ldg, weight,          \
                       static_cast<T*>(out), ld, size, eps, mode)
    if (dtype == CELEG_F32 && by_fours) NORM_GO(float, 4);
    else if (dtype == CELEG_F32) NORM_GO(float, 1);
    else if (by_fours) NORM_GO(bf16, 4);
    else NORM_GO(bf16, 1);
#undef NORM_GO
    return CELEG_LAUNCH_RESULT();
}
