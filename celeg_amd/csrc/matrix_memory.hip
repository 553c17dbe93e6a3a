// A recurrent mixer with a matrix of memory per head and exponential input gates (mLSTM).
//
// Per token and head, with query q (times dim^-1/2), key k, value v, log input gate i and log
// forget gate f (both bent to c tanh(z / c), f through log sigmoid):
//     m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n likewise with k alone
//     o = S^T q / (max(|n.q|, exp(-m')) + 1e-6),  m from 0
// then o / rms(o) per head, times a weight over all heads' values, times sigmoid(g).  S [dim, vdim],
// n [dim] and m live in the request's slot, in 32-bit.  Everything behind the projections is 32-bit.
//
// Kernels:
//  * mm_step: one new token of a request, everything in one pass over its state (a workgroup per
//    (row, head));
//  * for portions, chunks of 64 rows.  With F_t the sum of f over the chunk's rows up to t, b_s =
//    i_s - F_s, B_t = max of b_s over s <= t, and m0 the number m before the chunk, the running
//    maximum is m_t = F_t + top_t with top_t = max(m0, B_t), and row t reads
//        S_t^T q = exp(m0 - top_t) S_0^T q + sum_{s <= t} exp(b_s - top_t) (k_s.q) v_s,
//    so nothing in a chunk waits for the token before it:
//      mm_gates: F, b, B, m for all rows (wavefront scans in double precision; b and top leave as
//        two 32-bit numbers each, so that their difference keeps 32-bit precision however far F runs);
//      mm_chunk_state: what every chunk adds to the state, sum_s exp(b_s - top_last) k_s v_s^T;
//      mm_carry: the states in front of all chunks, and the request's new state;
//      mm_chunk_out: the rows' results, norm and gate.
//    All matrix work runs on the 32-bit matrix instruction (16x16x4).
#include "common.h"

namespace {

typedef float mm_f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 mm_bf16x4 __attribute__((ext_vector_type(4)));

#define MM_ROWS 64        // rows of a chunk
#define MM_GATE_WAVES 16
#define MM_TINY 1e-6f

// planes of the gates' numbers, [plane][head][row]
enum { MM_TOP_HI = 0, MM_TOP_LO, MM_IN_HI, MM_IN_LO, MM_CARRY, MM_FLOOR, MM_PLANES };

__device__ __forceinline__ float mm_bend(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float mm_log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float mm_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// four neighbouring values of a row (vec: they lie on a boundary of four), those from `live` on zero
__device__ __forceinline__ mm_f32x4 mm_load4(const float* p, int live, bool vec) {
    if (vec && live >= 4) return *reinterpret_cast<const mm_f32x4*>(p);
    mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (e < live) v[e] = p[e];
    return v;
}
__device__ __forceinline__ mm_f32x4 mm_load4(const bf16* p, int live, bool vec) {
    mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (vec && live >= 4) {
        const mm_bf16x4 b = *reinterpret_cast<const mm_bf16x4*>(p);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = static_cast<float>(b[e]);
        return v;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (e < live) v[e] = to_float(p[e]);
    return v;
}

// where everything lies: columns of the projections' rows, the slots' states, the sizes
struct MmArgs {
    const void* proj;
    int ld, col_q, col_k, col_v, col_g, col_i, col_f;
    const float *bias_i, *bias_f, *norm;
    float *S, *n, *m;
    size_t ldS, ldn, ldm;             // distance between slots
    const int *cu_seqlens, *seq_slot, *token_slot;
    float* planes;
    float *chunk_s, *chunk_n;         // [chunk][head][dim * vdim], [chunk][head][dim]
    void* out;
    int ldo;
    int first_seq, n_seqs, n_rows, H, D, V, vec;
    float cap, eps, q_scale;
};

// ---------------------------------------------------------------- one new token
// One workgroup per (row, head).  Threads are laid over (group of rows of S, VEC neighbouring columns).
#define MM_STEP_THREADS 256
template <typename T, int VEC>
__global__ __launch_bounds__(MM_STEP_THREADS) void mm_step_kernel(const MmArgs a) {
    extern __shared__ float mm_lds[];
    __shared__ float scratch[16];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, D = a.D, V = a.V;
    const int n_cols = V / VEC, groups = max(1, MM_STEP_THREADS / n_cols);
    float* qs = mm_lds;
    float* ks = qs + D;
    float* vs = ks + D;
    float* part = vs + V;             // [groups][V]
    const T* row = static_cast<const T*>(a.proj) + static_cast<size_t>(t) * a.ld;
    const size_t slot = static_cast<size_t>(a.token_slot[t]);
    float* m_at = a.m + slot * a.ldm + h;
    const float m_old = *m_at;
    const float log_in = mm_bend(to_float(row[a.col_i + h]) + a.bias_i[h], a.cap);
    const float log_keep = mm_log_sigmoid(mm_bend(to_float(row[a.col_f + h]) + a.bias_f[h], a.cap)) + m_old;
    const float m_new = fmaxf(log_keep, log_in);
    const float keep = expf(log_keep - m_new), write = expf(log_in - m_new);
    for (int d = tid; d < D; d += MM_STEP_THREADS) {
        qs[d] = to_float(row[a.col_q + h * D + d]) * a.q_scale;
        ks[d] = to_float(row[a.col_k + h * D + d]);
    }
    for (int j = tid; j < V; j += MM_STEP_THREADS) vs[j] = to_float(row[a.col_v + h * V + j]) * write;
    __syncthreads();
    if (tid == 0) *m_at = m_new;      // (every thread has read it)

    float* S = a.S + slot * a.ldS + static_cast<size_t>(h) * D * V;
    const int g = tid / n_cols;
    if (g < groups) {
        for (int c = tid % n_cols; c < n_cols; c += MM_STEP_THREADS) {
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
                    const mm_f32x4 x = *reinterpret_cast<const mm_f32x4*>(p);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) s[e] = x[e];
                } else {
                    s[0] = p[0];
                }
            };
            auto store = [&](int d, const float (&s)[VEC]) __attribute__((always_inline)) {
                float* p = S + static_cast<size_t>(d) * V + c * VEC;
                if (VEC == 4) *reinterpret_cast<mm_f32x4*>(p) = mm_f32x4{s[0], s[VEC > 1 ? 1 : 0], s[VEC > 2 ? 2 : 0], s[VEC > 3 ? 3 : 0]};
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
    float* n = a.n + slot * a.ldn + static_cast<size_t>(h) * D;
    float nq = 0.f;
    for (int d = tid; d < D; d += MM_STEP_THREADS) {
        const float x = fmaf(ks[d], write, keep * n[d]);
        n[d] = x;
        nq = fmaf(x, qs[d], nq);
    }
    nq = block_sum(nq, scratch);      // (its barriers also end the writing of `part`)
    const float inv = 1.0f / (fmaxf(fabsf(nq), expf(-m_new)) + MM_TINY);
    float sq = 0.f;
    for (int j = tid; j < V; j += MM_STEP_THREADS) {
        float o = 0.f;
        for (int u = 0; u < groups; ++u) o += part[static_cast<size_t>(u) * V + j];
        o *= inv;
        part[j] = o;                  // (this thread alone reads column j)
        sq = fmaf(o, o, sq);
    }
    sq = block_sum(sq, scratch);
    const float unit = 1.0f / sqrtf(sq / static_cast<float>(V) + a.eps);
    T* out = static_cast<T*>(a.out) + static_cast<size_t>(t) * a.ldo + static_cast<size_t>(h) * V;
    for (int j = tid; j < V; j += MM_STEP_THREADS)
        out[j] = from_float<T>(part[j] * unit * a.norm[h * V + j] * mm_sigmoid(to_float(row[a.col_g + h * V + j])));
}

// ---------------------------------------------------------------- portions: the gates
// One workgroup per (request, head); a wavefront takes a chunk of 64 rows, a round 16 chunks.
template <typename T>
__global__ __launch_bounds__(MM_GATE_WAVES * CELEG_WAVE) void mm_gates_kernel(const MmArgs a) {
    __shared__ double sum_s[MM_GATE_WAVES], best_s[MM_GATE_WAVES];
    const int s = a.first_seq + blockIdx.x, h = blockIdx.y, lane = threadIdx.x % CELEG_WAVE, wave = threadIdx.x / CELEG_WAVE;
    const int row0 = a.cu_seqlens[s], n = a.cu_seqlens[s + 1] - row0;
    if (n <= 0) return;
    float* m_at = a.m + static_cast<size_t>(a.seq_slot[s]) * a.ldm + h;
    double carried = static_cast<double>(*m_at);
    __syncthreads();
    const size_t plane = static_cast<size_t>(a.H) * a.n_rows;
    for (int base = 0; base < n; base += MM_GATE_WAVES * MM_ROWS) {
        const int r = base + wave * MM_ROWS + lane;
        const bool in = r < n;
        double F = 0.0, b = -INFINITY;
        if (in) {
            const T* row = static_cast<const T*>(a.proj) + static_cast<size_t>(row0 + r) * a.ld;
            b = static_cast<double>(mm_bend(to_float(row[a.col_i + h]) + a.bias_i[h], a.cap));
            F = static_cast<double>(mm_log_sigmoid(mm_bend(to_float(row[a.col_f + h]) + a.bias_f[h], a.cap)));
        }
#pragma unroll
        for (int off = 1; off < CELEG_WAVE; off <<= 1) {
            const double y = __shfl_up(F, off, CELEG_WAVE);
            if (lane >= off) F += y;
        }
        b -= F;
        double B = b;
#pragma unroll
        for (int off = 1; off < CELEG_WAVE; off <<= 1) {
            const double y = __shfl_up(B, off, CELEG_WAVE);
            if (lane >= off) B = fmax(B, y);
        }
        if (lane == CELEG_WAVE - 1) {      // (rows past the end add nothing: f = 0, b = -inf)
            sum_s[wave] = F;
            best_s[wave] = B;
        }
        __syncthreads();
        double m0 = carried, after = carried;
#pragma unroll
        for (int w = 0; w < MM_GATE_WAVES; ++w) {
            if (w == wave) m0 = after;
            after = sum_s[w] + fmax(after, best_s[w]);
        }
        carried = after;
        if (in) {
            const double top = fmax(m0, B);
            float* at = a.planes + static_cast<size_t>(h) * a.n_rows + row0 + r;
            const float top_hi = static_cast<float>(top), in_hi = static_cast<float>(b);
            at[MM_TOP_HI * plane] = top_hi;
            at[MM_TOP_LO * plane] = static_cast<float>(top - static_cast<double>(top_hi));
            at[MM_IN_HI * plane] = in_hi;
            at[MM_IN_LO * plane] = static_cast<float>(b - static_cast<double>(in_hi));
            at[MM_CARRY * plane] = expf(static_cast<float>(m0 - top));
            at[MM_FLOOR * plane] = expf(-static_cast<float>(F + top));
        }
        __syncthreads();
    }
    if (threadIdx.x == 0) *m_at = static_cast<float>(carried);
}

// which request and chunk of it: the chunks of the requests from first_seq on, one after the other
__device__ __forceinline__ bool mm_find_chunk(const MmArgs& a, int index, int& s, int& row0, int& rows) {
    int chunk = index;
    for (s = a.first_seq; s < a.n_seqs; ++s) {
        const int start = a.cu_seqlens[s], n = a.cu_seqlens[s + 1] - start;
        const int chunks = (n + MM_ROWS - 1) / MM_ROWS;
        if (chunk < chunks) {
            row0 = start + chunk * MM_ROWS;
            rows = min(MM_ROWS, n - chunk * MM_ROWS);
            return true;
        }
        chunk -= chunks;
    }
    return false;
}

// ---------------------------------------------------------------- portions: what a chunk adds
// One workgroup per (chunk, head, 64 columns of the state).
template <typename T>
__global__ __launch_bounds__(256) void mm_chunk_state_kernel(const MmArgs a) {
    extern __shared__ __attribute__((aligned(16))) float mm_lds[];
    const int D = a.D, V = a.V, Dp = (D + 15) & ~15, KROW = Dp + 4, VROW = 64 + 4;
    float* Ks = mm_lds;                       // [64][KROW], weighted
    float* Vs = Ks + MM_ROWS * KROW;          // [64][VROW]
    int s, row0, rows;
    if (!mm_find_chunk(a, blockIdx.x, s, row0, rows)) return;
    const int h = blockIdx.y, col0 = blockIdx.z * 64;
    const int tid = threadIdx.x, lane = tid % CELEG_WAVE, wave = tid / CELEG_WAVE, c = lane & 15, quad = lane >> 4;
    const size_t plane = static_cast<size_t>(a.H) * a.n_rows;
    const float* gates = a.planes + static_cast<size_t>(h) * a.n_rows + row0;
    const float top_hi = gates[MM_TOP_HI * plane + rows - 1], top_lo = gates[MM_TOP_LO * plane + rows - 1];
    const T* base = static_cast<const T*>(a.proj) + static_cast<size_t>(row0) * a.ld;
    for (int i = tid; i < MM_ROWS * (Dp / 4); i += 256) {
        const int r = i / (Dp / 4), d = 4 * (i % (Dp / 4));
        mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows) {
            const float w = expf((gates[MM_IN_HI * plane + r] - top_hi) + (gates[MM_IN_LO * plane + r] - top_lo));
            v = mm_load4(base + static_cast<size_t>(r) * a.ld + a.col_k + h * D + d, D - d, a.vec) * w;
        }
        *reinterpret_cast<mm_f32x4*>(Ks + r * KROW + d) = v;
    }
    for (int i = tid; i < MM_ROWS * 16; i += 256) {
        const int r = i / 16, j = 4 * (i % 16);
        mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows) v = mm_load4(base + static_cast<size_t>(r) * a.ld + a.col_v + h * V + col0 + j, V - col0 - j, a.vec);
        *reinterpret_cast<mm_f32x4*>(Vs + r * VROW + j) = v;
    }
    __syncthreads();
    const size_t at = static_cast<size_t>(blockIdx.x) * a.H + h;
    if (blockIdx.z == 0)
        for (int d = tid; d < D; d += 256) {
            float sum = 0.f;
            for (int r = 0; r < rows; ++r) sum += Ks[r * KROW + d];
            a.chunk_n[at * D + d] = sum;
        }
    float* out = a.chunk_s + at * D * V;
    const int groups = (rows + 15) / 16;
    for (int dt = wave; dt < Dp / 16; dt += 4) {
        mm_f32x4 acc[4];
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) acc[ct] = mm_f32x4{0.f, 0.f, 0.f, 0.f};
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

// ---------------------------------------------------------------- portions: the states in front of the chunks
// A thread per number of (S | n) and (request, head): chunk by chunk, what the chunk adds makes room for
// the state in front of it; what is left at the end is the request's new state.
__global__ __launch_bounds__(256) void mm_carry_kernel(const MmArgs a) {
    const int e = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, s = a.first_seq + blockIdx.z;
    const int per_s = a.D * a.V;
    if (e >= per_s + a.D) return;
    int chunk0 = 0;
    for (int p = a.first_seq; p < s; ++p) chunk0 += (a.cu_seqlens[p + 1] - a.cu_seqlens[p] + MM_ROWS - 1) / MM_ROWS;
    const int row0 = a.cu_seqlens[s], n = a.cu_seqlens[s + 1] - row0;
    if (n <= 0) return;
    const size_t slot = static_cast<size_t>(a.seq_slot[s]);
    const bool is_s = e < per_s;
    float* mine = is_s ? a.S + slot * a.ldS + static_cast<size_t>(h) * per_s + e : a.n + slot * a.ldn + static_cast<size_t>(h) * a.D + (e - per_s);
    const size_t step = static_cast<size_t>(a.H) * (is_s ? per_s : a.D);
    float* at = (is_s ? a.chunk_s + (static_cast<size_t>(chunk0) * a.H + h) * per_s + e
                      : a.chunk_n + (static_cast<size_t>(chunk0) * a.H + h) * a.D + (e - per_s));
    const float* carry = a.planes + static_cast<size_t>(MM_CARRY) * a.H * a.n_rows + static_cast<size_t>(h) * a.n_rows + row0;
    float x = *mine;
    const int chunks = (n + MM_ROWS - 1) / MM_ROWS;
    int i = 0;
    for (; i + 8 <= chunks; i += 8) {
        float added[8], keep[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            added[u] = at[(i + u) * step];
            keep[u] = carry[min((i + u + 1) * MM_ROWS, n) - 1];
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
        x = fmaf(carry[min((i + 1) * MM_ROWS, n) - 1], x, added);
    }
    *mine = x;
}

// ---------------------------------------------------------------- portions: the rows' results
// One workgroup of four wavefronts per (chunk, head), 16 rows a wavefront.  KG: groups of 16 key
// numbers, VT: tiles of 16 value columns (upper bounds of the head's sizes).
template <typename T, int KG, int VT>
__global__ __launch_bounds__(256) void mm_chunk_out_kernel(const MmArgs a) {
    extern __shared__ __attribute__((aligned(16))) float mm_lds[];
    const int D = a.D, V = a.V, Dp = (D + 15) & ~15, KROW = Dp + 4;
    constexpr int PROW = MM_ROWS + 4, VROW = 64 + 4;
    float* Ks = mm_lds;                              // [64][KROW]
    float* Vs = Ks + MM_ROWS * KROW;                 // [64][VROW]
    float* Ps = Vs + MM_ROWS * VROW;                 // [4][16][PROW]
    float* Qn = Ps + 4 * 16 * PROW;                  // [4][16]
    int s, row0, rows;
    if (!mm_find_chunk(a, blockIdx.x, s, row0, rows)) return;
    const int h = blockIdx.y, tid = threadIdx.x, lane = tid % CELEG_WAVE, wave = tid / CELEG_WAVE, c = lane & 15, quad = lane >> 4;
    const size_t plane = static_cast<size_t>(a.H) * a.n_rows;
    const float* gates = a.planes + static_cast<size_t>(h) * a.n_rows + row0;
    const T* base = static_cast<const T*>(a.proj) + static_cast<size_t>(row0) * a.ld;
    const size_t at = static_cast<size_t>(blockIdx.x) * a.H + h;
    const float* S0 = a.chunk_s + at * D * V;
    const float* n0 = a.chunk_n + at * D;
    const bool vec = a.vec != 0;

    // this wavefront's queries: lane (c, quad) holds numbers 16 g + 4 quad .. + 3 of row 16 wave + c
    const int q_row = 16 * wave + c;
    mm_f32x4 q[KG];
    float qn = 0.f;
#pragma unroll
    for (int g = 0; g < KG; ++g) {
        const int d = 16 * g + 4 * quad;
        q[g] = mm_f32x4{0.f, 0.f, 0.f, 0.f};
        if (d < D && q_row < rows) {
            q[g] = mm_load4(base + static_cast<size_t>(q_row) * a.ld + a.col_q + h * D + d, D - d, vec) * a.q_scale;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (d + e < D) qn = fmaf(q[g][e], n0[d + e], qn);
        }
    }
    qn += __shfl_xor(qn, 16, CELEG_WAVE);
    qn += __shfl_xor(qn, 32, CELEG_WAVE);
    if (quad == 0) Qn[16 * wave + c] = qn;
    for (int i = tid; i < MM_ROWS * (Dp / 4); i += 256) {
        const int r = i / (Dp / 4), d = 4 * (i % (Dp / 4));
        mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < rows) v = mm_load4(base + static_cast<size_t>(r) * a.ld + a.col_k + h * D + d, D - d, vec);
        *reinterpret_cast<mm_f32x4*>(Ks + r * KROW + d) = v;
    }
    __syncthreads();

    // the numbers of this lane's result rows, 16 wave + 4 quad + i
    float top_hi[4], top_lo[4], carry[4], denom[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = min(16 * wave + 4 * quad + i, rows - 1);
        top_hi[i] = gates[MM_TOP_HI * plane + t];
        top_lo[i] = gates[MM_TOP_LO * plane + t];
        carry[i] = gates[MM_CARRY * plane + t];
    }
    float total[4] = {0.f, 0.f, 0.f, 0.f};
    float* mine = Ps + wave * 16 * PROW;
    for (int st = 0; st <= wave; ++st) {              // keys behind the wavefront's last row are not seen
        mm_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int g = 0; g < KG; ++g)
            if (16 * g < D) {
                const mm_f32x4 k = *reinterpret_cast<const mm_f32x4*>(Ks + (16 * st + c) * KROW + 16 * g + 4 * quad);
#pragma unroll
                for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q[g][e], k[e], acc, 0, 0, 0);
            }
        const int key = 16 * st + c, safe = min(key, rows - 1);
        const float in_hi = gates[MM_IN_HI * plane + safe], in_lo = gates[MM_IN_LO * plane + safe];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * quad + i;
            const float w = key <= t && key < rows ? acc[i] * expf((in_hi - top_hi[i]) + (in_lo - top_lo[i])) : 0.f;
            mine[(4 * quad + i) * PROW + key] = w;
            total[i] += w;
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * quad + i;
        const float nq = fmaf(carry[i], Qn[t], lanes_sum<16>(total[i]));
        denom[i] = 1.0f / (fmaxf(fabsf(nq), gates[MM_FLOOR * plane + min(t, rows - 1)]) + MM_TINY);
    }
    mm_f32x4 o[VT];
    float sq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ct = 0; ct < VT; ++ct) {
        if (16 * ct >= V) continue;                   // (the same for every thread)
        if (ct % 4 == 0) {
            __syncthreads();
            for (int i = tid; i < MM_ROWS * 16; i += 256) {
                const int r = i / 16, j = 16 * ct + 4 * (i % 16);
                mm_f32x4 v = {0.f, 0.f, 0.f, 0.f};
                if (r < rows && j < V) v = mm_load4(base + static_cast<size_t>(r) * a.ld + a.col_v + h * V + j, V - j, vec);
                *reinterpret_cast<mm_f32x4*>(Vs + r * VROW + 4 * (i % 16)) = v;
            }
            __syncthreads();
        }
        const int j = 16 * ct + c;
        const bool has = j < V;
        mm_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
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
            const mm_f32x4 p = *reinterpret_cast<const mm_f32x4*>(mine + c * PROW + 16 * g + 4 * quad);
#pragma unroll
            for (int e = 0; e < 4; ++e)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(p[e], Vs[(16 * g + 4 * quad + e) * VROW + 16 * (ct % 4) + c], acc, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            o[ct][i] = acc[i] * denom[i];
            sq[i] = fmaf(o[ct][i], o[ct][i], sq[i]);  // (columns past the head's are zero)
        }
    }
    float unit[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) unit[i] = 1.0f / sqrtf(lanes_sum<16>(sq[i]) / static_cast<float>(V) + a.eps);
#pragma unroll
    for (int ct = 0; ct < VT; ++ct) {
        const int j = 16 * ct + c;
        if (j >= V) continue;
        const float w = a.norm[h * V + j];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * quad + i;
            if (t >= rows) continue;
            const float z = to_float(base[static_cast<size_t>(t) * a.ld + a.col_g + h * V + j]);
            static_cast<T*>(a.out)[static_cast<size_t>(row0 + t) * a.ldo + static_cast<size_t>(h) * V + j] =
                from_float<T>(o[ct][i] * unit[i] * w * mm_sigmoid(z));
        }
    }
}

int mm_allow(const void* kernel, size_t lds) {
    if (lds <= 64 * 1024) return 0;
    return static_cast<int>(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)));
}

template <typename T, int KG, int VT>
int mm_out_launch(const MmArgs& a, int max_chunks, size_t lds, hipStream_t stream) {
    auto kernel = mm_chunk_out_kernel<T, KG, VT>;
    if (int rc = mm_allow(reinterpret_cast<const void*>(kernel), lds)) return rc;
    hipLaunchKernelGGL(kernel, dim3(max_chunks, a.H), dim3(256), lds, stream, a);
    return CELEG_LAUNCH_RESULT();
}
template <typename T, int KG>
int mm_out_launch_v(const MmArgs& a, int max_chunks, size_t lds, hipStream_t stream) {
    const int tiles = (a.V + 15) / 16;
    if (tiles <= 4) return mm_out_launch<T, KG, 4>(a, max_chunks, lds, stream);
    if (tiles <= 8) return mm_out_launch<T, KG, 8>(a, max_chunks, lds, stream);
    if (tiles <= 16) return mm_out_launch<T, KG, 16>(a, max_chunks, lds, stream);
    return mm_out_launch<T, KG, 32>(a, max_chunks, lds, stream);
}

template <typename T>
int mm_rows(const MmArgs& a, int max_chunks, hipStream_t stream) {
    const int Dp = (a.D + 15) & ~15, seqs = a.n_seqs - a.first_seq;
    hipLaunchKernelGGL(mm_gates_kernel<T>, dim3(seqs, a.H), dim3(MM_GATE_WAVES * CELEG_WAVE), 0, stream, a);
    if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    const size_t state_lds = (static_cast<size_t>(MM_ROWS) * (Dp + 4) + MM_ROWS * 68) * sizeof(float);
    if (int rc = mm_allow(reinterpret_cast<const void*>(mm_chunk_state_kernel<T>), state_lds)) return rc;
    hipLaunchKernelGGL(mm_chunk_state_kernel<T>, dim3(max_chunks, a.H, (a.V + 63) / 64), dim3(256), state_lds, stream, a);
    if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    hipLaunchKernelGGL(mm_carry_kernel, dim3((a.D * a.V + a.D + 255) / 256, a.H, seqs), dim3(256), 0, stream, a);
    if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    const size_t out_lds = (static_cast<size_t>(MM_ROWS) * (Dp + 4) + MM_ROWS * 68 + 4 * 16 * (MM_ROWS + 4) + 64) * sizeof(float);
    if (Dp <= 64) return mm_out_launch_v<T, 4>(a, max_chunks, out_lds, stream);
    if (Dp <= 128) return mm_out_launch_v<T, 8>(a, max_chunks, out_lds, stream);
    return mm_out_launch_v<T, 16>(a, max_chunks, out_lds, stream);
}

}  // namespace

// proj [rows, ld]: q and k (heads x dim) at col_q and col_k, v and the output gate (heads x vdim) at col_v
// and col_g, the gates' inputs (heads) at col_i and col_f.  Rows [0, n_single) are requests of one new token;
// the requests from n_single on bring portions, whose chunks of 64 rows are at most max_chunks.  planes: room for
// 6 * heads * n_rows numbers, chunk_s for max_chunks * heads * dim * vdim, chunk_n for max_chunks * heads * dim.
extern "C" int celeg_matrix_memory(const void* proj, int ld, int dtype, int col_q, int col_k, int col_v, int col_g, int col_i, int col_f,
                                   const float* bias_i, const float* bias_f, const float* norm, float* S, size_t ldS, float* n,
                                   size_t ldn, float* m, size_t ldm, const int* cu_seqlens, const int* seq_slot, const int* token_slot,
                                   float* planes, float* chunk_s, float* chunk_n, void* out, int ldo, int n_rows, int n_seqs,
                                   int n_single, int max_chunks, int H, int D, int V, float cap, float eps, hipStream_t stream) {
    if (n_rows <= 0 || n_seqs <= 0) return 0;
    if (H <= 0 || D <= 0 || V <= 0 || D > 256 || V > 512 || n_single < 0 || n_single > n_seqs || !(cap > 0.f))
        return static_cast<int>(hipErrorInvalidValue);
    MmArgs a;
    a.proj = proj;
    a.ld = ld;
    a.col_q = col_q;
    a.col_k = col_k;
    a.col_v = col_v;
    a.col_g = col_g;
    a.col_i = col_i;
    a.col_f = col_f;
    a.bias_i = bias_i;
    a.bias_f = bias_f;
    a.norm = norm;
    a.S = S;
    a.n = n;
    a.m = m;
    a.ldS = ldS;
    a.ldn = ldn;
    a.ldm = ldm;
    a.cu_seqlens = cu_seqlens;
    a.seq_slot = seq_slot;
    a.token_slot = token_slot;
    a.planes = planes;
    a.chunk_s = chunk_s;
    a.chunk_n = chunk_n;
    a.out = out;
    a.ldo = ldo;
    a.first_seq = n_single;
    a.n_seqs = n_seqs;
    a.n_rows = n_rows;
    a.H = H;
    a.D = D;
    a.V = V;
    a.cap = cap;
    a.eps = eps;
    a.q_scale = 1.0f / sqrtf(static_cast<float>(D));
    const size_t four = dtype == CELEG_F32 ? 16 : 8;
    a.vec = ((ld | col_q | col_k | col_v | D | V) & 3) == 0 && (reinterpret_cast<uintptr_t>(proj) & (four - 1)) == 0;
    if (n_single > 0) {
        // four columns a thread where the states allow it
        const bool by_fours = V % 4 == 0 && ldS % 4 == 0 && (reinterpret_cast<uintptr_t>(S) & 15) == 0;
        const int n_cols = by_fours ? V / 4 : V, groups = n_cols >= MM_STEP_THREADS ? 1 : MM_STEP_THREADS / n_cols;
        const size_t lds = (2 * static_cast<size_t>(D) + V + static_cast<size_t>(groups) * V) * sizeof(float);
        dim3 grid(n_single, H), block(MM_STEP_THREADS);
        if (dtype == CELEG_F32 && by_fours) hipLaunchKernelGGL((mm_step_kernel<float, 4>), grid, block, lds, stream, a);
        else if (dtype == CELEG_F32) hipLaunchKernelGGL((mm_step_kernel<float, 1>), grid, block, lds, stream, a);
        else if (by_fours) hipLaunchKernelGGL((mm_step_kernel<bf16, 4>), grid, block, lds, stream, a);
        else hipLaunchKernelGGL((mm_step_kernel<bf16, 1>), grid, block, lds, stream, a);
        if (int rc = CELEG_LAUNCH_RESULT()) return rc;
    }
    if (n_seqs == n_single) return 0;
    if (max_chunks <= 0 || !planes || !chunk_s || !chunk_n) return static_cast<int>(hipErrorInvalidValue);
    return dtype == CELEG_F32 ? mm_rows<float>(a, max_chunks, stream) : mm_rows<bf16>(a, max_chunks, stream);
}
