// Matrix memory with exponential gates (mLSTM), for batches of portions of sequences.  A head keeps a matrix
// S [key channels x value channels], a vector n [key channels] and the running maximum m of the log gates, all
// float, in the request's slot; with q scaled by `q_scale`, and per token the log input gate i and log forget gate f,
//
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- e^(f + m - m') n + e^(i - m') k
//   o = S^T q / (max(|n . q|, e^(-m')) + 1e-6)
//   i = cap tanh((zi + bi) / cap);   f = log sigmoid(cap tanh((zf + bf) / cap))
//   y = o / sqrt(mean(o^2) + eps) * gain * sigmoid(g)          per head, gain and g [heads x value channels]
//
// Two routes over one state.  A step of single tokens is one kernel (`step`), a workgroup a head and request:
// gates, state, read-out, norm and gate.  Other steps go by chunks of 64 rows, counted from an item's first row of
// the step, with products on the matrix cores in float.  With F_j the sum of f over a chunk's rows up to j (double: the
// sums cancel in the exponents), c_j = i_j - F_j and M_j = max(m_0, c_0 .. c_j), the recurrence from the state
// (S_0, n_0, m_0) of the chunk's start is, all exponents being <= 0,
//
//   m_j = F_j + M_j,   S_j = e^(m_0 - M_j) S_0 + sum_(l <= j) e^(c_l - M_j) k_l v_l^T,   n_j likewise
//
// so a chunk's own sums, taken relative to its own largest c, need no state and the chunks run side by side
// (`sums`); `carry` walks a request's chunks and leaves each one's start state in its sums' place; `outputs` forms
// the rows' results with norm and gate.
//
// A row of `proj` is q | k | v | g | zi | zf: (heads x dk) twice, (heads x dv) twice, heads twice, floats.
// A slot is S [heads, dk, dv] | n [heads, dk] | m [heads].
#include "api.h"
#include "chunk_tiles.h"
#include "common.h"

#include <mutex>
#include <set>

namespace st {

typedef float floatx4 __attribute__((ext_vector_type(4)));

constexpr int kMemChunk = kChunkRows;
constexpr int kMemMaxDim = 256;

__device__ inline float log_input_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ inline float log_forget_gate(float z, float cap) {
    const float u = cap * tanhf(z / cap);
    return fminf(u, 0.f) - log1pf(expf(-fabsf(u)));
}

struct MemoryShape {
    int heads, dk, dv;
    __host__ __device__ int64_t k_off() const { return (int64_t)heads * dk; }
    __host__ __device__ int64_t v_off() const { return 2 * (int64_t)heads * dk; }
    __host__ __device__ int64_t g_off() const { return 2 * (int64_t)heads * dk + (int64_t)heads * dv; }
    __host__ __device__ int64_t i_off() const { return 2 * (int64_t)heads * (dk + dv); }
    __host__ __device__ int64_t f_off() const { return i_off() + heads; }
    __host__ __device__ int64_t row() const { return i_off() + 2 * heads; }
    __host__ __device__ int64_t n_base() const { return (int64_t)heads * dk * dv; }
    __host__ __device__ int64_t m_base() const { return n_base() + (int64_t)heads * dk; }
    __host__ __device__ int64_t slot() const { return m_base() + heads; }
};

// ---------------------------------------------------------------- single tokens
// A workgroup a (head, item).  A thread owns V neighbouring value channels and every `lanes`-th key channel; the
// state travels in batches of 8 such pieces, all asked for at once.  LDS: q | k [dk] | o partial sums [lanes][dv] | red.
template <typename T, int V>
__global__ __launch_bounds__(1024) void memory_step_kernel(
    T* __restrict__ out, const float* __restrict__ proj, int64_t stride, float* __restrict__ state, int64_t slot_stride,
    const float* __restrict__ bias_i, const float* __restrict__ bias_f, const float* __restrict__ gain,
    const int* __restrict__ item_len, const int* __restrict__ item_tok_off, const int* __restrict__ item_slot,
    MemoryShape sh, float cap, float q_scale, float eps, int lanes) {
    extern __shared__ __attribute__((aligned(16))) float mem_lds[];
    const int head = blockIdx.x, item = blockIdx.y, tid = threadIdx.x;
    const int slot = item_slot[item];
    if (slot < 0 || item_len[item] <= 0) return;
    const int dk = sh.dk, dv = sh.dv, cols = dv / V;
    const int64_t row = item_tok_off[item];
    const float* p = proj + row * stride;
    float* sl = state + (int64_t)slot * slot_stride;
    float* S = sl + (int64_t)head * dk * dv;
    float* nv = sl + sh.n_base() + (int64_t)head * dk;
    float* mp = sl + sh.m_base() + head;
    float* sq = mem_lds;
    float* sk = sq + dk;
    float* part = sk + dk;
    float* red = part + lanes * dv;
    const int c = tid % cols, kl = tid / cols;
    const bool works = kl < lanes;
    constexpr int B = 8;
    // asked for at once: gates, m, q, k, n, v and the first batch of the state
    const float zi = p[sh.i_off() + head] + bias_i[head], zf = p[sh.f_off() + head] + bias_f[head];
    const float m_old = *mp;
    float qv = 0.f, kv = 0.f, n_old = 0.f;
    if (tid < dk) {
        qv = p[(int64_t)head * dk + tid] * q_scale;
        kv = p[sh.k_off() + (int64_t)head * dk + tid];
        n_old = nv[tid];
    }
    float v[V], s[B][V];
    if (works) {
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] = p[sh.v_off() + (int64_t)head * dv + c * V + e];
    }
    auto load = [&](int base) {
#pragma unroll
        for (int b = 0; b < B; ++b) {
            const int kk = min(base + b * lanes + kl, dk - 1);
            const float* src = S + (int64_t)kk * dv + c * V;
            if (V == 4) {
                const float4 x = *reinterpret_cast<const float4*>(src);
                s[b][0] = x.x; s[b][1 % V] = x.y; s[b][2 % V] = x.z; s[b][3 % V] = x.w;
            } else {
                s[b][0] = src[0];
            }
        }
    };
    if (works) load(0);
    const float gi = log_input_gate(zi, cap), gf = log_forget_gate(zf, cap);
    const float m_new = fmaxf(gf + m_old, gi);
    const float keep = expf(gf + m_old - m_new), add = expf(gi - m_new);
    if (tid < dk) { sq[tid] = qv; sk[tid] = kv; }
    __syncthreads();
    float acc[V];
#pragma unroll
    for (int e = 0; e < V; ++e) acc[e] = 0.f;
    if (works) {
        for (int base = 0; base < dk; base += B * lanes) {
            if (base) load(base);
#pragma unroll
            for (int b = 0; b < B; ++b) {
                const int kk = base + b * lanes + kl;
                if (kk >= dk) continue;
                const float kw = sk[kk] * add, qk = sq[kk];
                float* dst = S + (int64_t)kk * dv + c * V;
#pragma unroll
                for (int e = 0; e < V; ++e) {
                    s[b][e] = fmaf(keep, s[b][e], kw * v[e]);
                    acc[e] = fmaf(s[b][e], qk, acc[e]);
                }
                if (V == 4) *reinterpret_cast<float4*>(dst) = make_float4(s[b][0], s[b][1 % V], s[b][2 % V], s[b][3 % V]);
                else dst[0] = s[b][0];
            }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) part[kl * dv + c * V + e] = acc[e];
    }
    float den = 0.f;
    if (tid < dk) {
        const float n_new = fmaf(keep, n_old, add * kv);
        nv[tid] = n_new;
        den = n_new * qv;
    }
    den = block_sum(den, red);                     // (its barriers also order the partial sums)
    if (tid == 0) *mp = m_new;                     // every thread has read the old one
    den = fmaxf(fabsf(den), expf(-m_new)) + 1e-6f;
    float o = 0.f;
    if (tid < dv) {
        for (int j = 0; j < lanes; ++j) o += part[j * dv + tid];
        o /= den;
    }
    const float ss = block_sum(o * o, red);
    if (tid < dv) {
        const int64_t at = (int64_t)head * dv + tid;
        const float z = p[sh.g_off() + at];
        const float y = o / sqrtf(ss / (float)dv + eps) * gain[at] / (1.f + expf(-z));
        Elem<T>::store(out + row * ((int64_t)sh.heads * dv) + at, y);
    }
}

// ---------------------------------------------------------------- chunks
// The first wave: F_j (inclusive sums of the log forget gates) and c_j = i_j - F_j of a chunk's n rows; c = -inf past
// them.  `last`: the chunk's whole sum F_(n-1).
__device__ inline void memory_chunk_gates(double& F, double& c, double& last, const float* __restrict__ p, int64_t stride,
                                          const float* __restrict__ bias_i, const float* __restrict__ bias_f,
                                          const MemoryShape& sh, int head, int n, float cap) {
    const int lane = threadIdx.x & 63;
    double gi = 0.0;
    F = 0.0;
    if (lane < n) {
        const float* r = p + (int64_t)lane * stride;
        gi = (double)log_input_gate(r[sh.i_off() + head] + bias_i[head], cap);
        F = (double)log_forget_gate(r[sh.f_off() + head] + bias_f[head], cap);
    }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const double up = __shfl_up(F, o, 64);
        if (lane >= o) F += up;
    }
    last = __shfl(F, n - 1, 64);
    c = lane < n ? gi - F : -INFINITY;
}

__device__ inline double wave_max_double(double v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmax(v, __shfl_xor(v, o, 64));
    return v;
}

// U[idx, head] = sum_j e^(c_j - max c) k_j v_j^T [dk, dv], N[idx, head] the same sum of k_j, scal[idx, head] =
// (F of the whole chunk, max c).  Grid (heads, chunks, blocks of 64 value channels); a wave takes rows of 16 x 16 tiles.
// KQ: dk <= 4 KQ.  LDS: k [64][4 KQ + 4] (weighted), v [64][68], weights [64].  A matrix instruction sums 4 keys: lane
// group g of step (s, r) takes key 16 s + 4 g + r, which spreads its reads over the banks.
template <int KQ, bool VEC>
__global__ __launch_bounds__(256) void memory_sums_kernel(
    float* __restrict__ U, float* __restrict__ N, double* __restrict__ scal, const float* __restrict__ proj, int64_t stride,
    const float* __restrict__ bias_i, const float* __restrict__ bias_f, const int* __restrict__ item_len,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int num_items, MemoryShape sh, float cap) {
    extern __shared__ __attribute__((aligned(16))) float mem_lds[];
    const int head = blockIdx.x, idx = blockIdx.y, vb = blockIdx.z * 64, tid = threadIdx.x;
    int item, chunk;
    if (!find_chunk(idx, item_len, item_slot, num_items, item, chunk)) return;
    const int n = min(kMemChunk, item_len[item] - chunk * kMemChunk);
    const int64_t row0 = (int64_t)item_tok_off[item] + (int64_t)chunk * kMemChunk;
    const float* p = proj + row0 * stride;
    const int dk = sh.dk, dv = sh.dv, ktiles = (dk + 15) >> 4;
    constexpr int KS = 4 * KQ + 4, VS = 68;
    float* ks = mem_lds;
    float* vs = ks + kMemChunk * KS;
    float* w = vs + kMemChunk * VS;
    Tile<KQ> tk;
    Tile<16> tv;
    tk.template load<VEC>(p + sh.k_off() + (int64_t)head * dk, stride, n, 0, dk);
    tv.template load<VEC>(p + sh.v_off() + (int64_t)head * dv, stride, n, vb, dv);
    if (tid < 64) {
        double F, c, last;
        memory_chunk_gates(F, c, last, p, stride, bias_i, bias_f, sh, head, n, cap);
        const double mx = wave_max_double(c);
        w[tid] = tid < n ? expf((float)(c - mx)) : 0.f;
        if (blockIdx.z == 0 && tid == 0) {
            scal[((int64_t)idx * sh.heads + head) * 2] = last;
            scal[((int64_t)idx * sh.heads + head) * 2 + 1] = mx;
        }
    }
    tv.store(vs, VS);
    __syncthreads();                                // the weights
    tk.store_weighted(ks, KS, w);
    __syncthreads();
    const int lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int steps = (n + 15) >> 4;                // 16 keys each
    float* u = U + ((int64_t)idx * sh.heads + head) * dk * dv;
    const bool with_n = blockIdx.z == 0;
    for (int kt = wave; kt < ktiles; kt += 4) {
        floatx4 acc[4], an = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int vt = 0; vt < 4; ++vt) acc[vt] = floatx4{0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < steps; ++s) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = 16 * s + 4 * g + r;
                const float a = ks[j * KS + 16 * kt + r16];
                if (with_n) an = __builtin_amdgcn_mfma_f32_16x16x4f32(a, 1.f, an, 0, 0, 0);
#pragma unroll
                for (int vt = 0; vt < 4; ++vt)
                    acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vs[j * VS + 16 * vt + r16], acc[vt], 0, 0, 0);
            }
        }
        // acc[vt][r]: key channel 16 kt + 4 g + r, value channel 16 vt + r16
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int kk = 16 * kt + 4 * g + r;
            if (kk >= dk) continue;
            if (with_n && r16 == 0) N[((int64_t)idx * sh.heads + head) * dk + kk] = an[r];
#pragma unroll
            for (int vt = 0; vt < 4; ++vt) {
                const int col = vb + 16 * vt + r16;
                if (col < dv) u[(int64_t)kk * dv + col] = acc[vt][r];
            }
        }
    }
}

// A thread an element of (S | n) of a head walks the request's chunks: each chunk's sums make room for the state it
// starts from, and start_m receives its m; the last S and n go back to the slot (m follows with the outputs).
__global__ __launch_bounds__(256) void memory_carry_kernel(
    float* __restrict__ U, float* __restrict__ N, const double* __restrict__ scal, float* __restrict__ start_m,
    float* __restrict__ state, int64_t slot_stride, const int* __restrict__ item_len, const int* __restrict__ item_slot,
    MemoryShape sh) {
    const int head = blockIdx.x, item = blockIdx.y;
    const int slot = item_slot[item], len = item_len[item];
    const int plane = sh.dk * sh.dv;
    const int e = blockIdx.z * 256 + threadIdx.x;
    if (slot < 0 || len <= 0 || e >= plane + sh.dk) return;
    int base = 0;
    for (int b = 0; b < item; ++b) {
        const int l = item_len[b];
        base += (item_slot[b] >= 0 && l > 0) ? (l + kMemChunk - 1) / kMemChunk : 0;
    }
    const int chunks = (len + kMemChunk - 1) / kMemChunk;
    float* sl = state + (int64_t)slot * slot_stride;
    const bool in_n = e >= plane;
    float* home = in_n ? sl + sh.n_base() + (int64_t)head * sh.dk + (e - plane) : sl + (int64_t)head * plane + e;
    const int64_t first = (int64_t)base * sh.heads + head;
    float* u = in_n ? N + first * sh.dk + (e - plane) : U + first * plane + e;
    const int64_t step = (int64_t)sh.heads * (in_n ? sh.dk : plane);
    const double* sc = scal + first * 2;
    float S = *home;
    double m = (double)sl[sh.m_base() + head];
    constexpr int B = 16;                           // chunks asked for at once
    for (int c0 = 0; c0 < chunks; c0 += B) {
        float add[B];
        double total[B], mx[B];
#pragma unroll
        for (int b = 0; b < B; ++b) {
            const int64_t c = min(c0 + b, chunks - 1);
            add[b] = u[c * step];
            total[b] = sc[c * 2 * sh.heads];
            mx[b] = sc[c * 2 * sh.heads + 1];
        }
#pragma unroll
        for (int b = 0; b < B; ++b) {
            if (c0 + b >= chunks) continue;
            u[(int64_t)(c0 + b) * step] = S;
            if (e == 0) start_m[first + (int64_t)(c0 + b) * sh.heads] = (float)m;
            const double top = fmax(m, mx[b]);
            S = expf((float)(m - top)) * S + expf((float)(mx[b] - top)) * add[b];
            m = (double)(float)(total[b] + top);
        }
    }
    *home = S;
}

// Rows of a chunk, transposed: S^T = K Q^T leaves a lane with keys 4 g + r of ONE row (lane % 16), so weights, the
// denominator and the norm are per-lane numbers and sums over the four lane groups, and the weighted scores are the
// next product's operand as they lie (O^T += V^T P^T, 4 keys an instruction: key 4 g + r of lane group g).  Key channel
// 4 s + g belongs to lane group g in step s of the products over key channels.
// Four waves, 16 rows each.  NV: tiles of 16 value channels (dv <= 16 NV); KQ: dk <= 4 KQ.
// LDS: c, M doubles [64] each | m [64] | k [64][4 KQ + 4], later 64 key channels of the start state [64][16 NV + 16] |
// v [64][16 NV + 4]: strides that spread the instructions' reads over the banks.
template <int KQ, int NV>
struct MemoryOutLds {
    static constexpr int KS = 4 * KQ + 4, VS = 16 * NV + 4, SS = 16 * NV + 16;
    static constexpr int first = KS > SS ? 64 * KS : 64 * SS;
    static constexpr size_t bytes = sizeof(double) * 2 * kMemChunk + sizeof(float) * (size_t)(kMemChunk + first + 64 * VS);
};

template <typename T, int KQ, int NV, bool VEC>
__global__ __launch_bounds__(256) void memory_out_kernel(
    T* __restrict__ out, const float* __restrict__ proj, int64_t stride, float* __restrict__ state, int64_t slot_stride,
    const float* __restrict__ S0, const float* __restrict__ N0, const float* __restrict__ start_m,
    const float* __restrict__ bias_i, const float* __restrict__ bias_f, const float* __restrict__ gain,
    const int* __restrict__ item_len, const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int num_items,
    MemoryShape sh, float cap, float q_scale, float eps) {
    extern __shared__ __attribute__((aligned(16))) float mem_lds[];
    using L = MemoryOutLds<KQ, NV>;
    const int head = blockIdx.x, idx = blockIdx.y, tid = threadIdx.x;
    int item, chunk;
    if (!find_chunk(idx, item_len, item_slot, num_items, item, chunk)) return;
    const int n = min(kMemChunk, item_len[item] - chunk * kMemChunk);
    const int64_t row0 = (int64_t)item_tok_off[item] + (int64_t)chunk * kMemChunk;
    const float* p = proj + row0 * stride;
    const int dk = sh.dk, dv = sh.dv;
    double* sc = reinterpret_cast<double*>(mem_lds);           // c_j
    double* sM = sc + kMemChunk;                               // M_j
    float* sm = reinterpret_cast<float*>(sM + kMemChunk);      // m_j = F_j + M_j
    float* ks = sm + kMemChunk;
    float* vs = ks + L::first;
    const int64_t at = (int64_t)idx * sh.heads + head;
    const int lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int i = wave * 16 + r16;                             // this lane's row of the chunk
    const bool row_ok = i < n;
    const float m0 = start_m[at];
    {
        Tile<KQ> tk;
        Tile<4 * NV> tv;
        tk.template load<VEC>(p + sh.k_off() + (int64_t)head * dk, stride, n, 0, dk);
        tv.template load<VEC>(p + sh.v_off() + (int64_t)head * dv, stride, n, 0, dv);
        if (tid < 64) {
            double F, c, last;
            memory_chunk_gates(F, c, last, p, stride, bias_i, bias_f, sh, head, n, cap);
            double M = c;
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const double up = __shfl_up(M, o, 64);
                if (tid >= o) M = fmax(M, up);
            }
            M = fmax(M, (double)m0);
            sc[tid] = c;
            sM[tid] = M;
            sm[tid] = (float)(F + M);
            // the request's last row leaves its maximum in the slot (the carry has read the old one)
            if (tid == n - 1 && (chunk + 1) * kMemChunk >= item_len[item])
                state[(int64_t)item_slot[item] * slot_stride + sh.m_base() + head] = (float)(F + M);
        }
        tk.store(ks, L::KS);
        tv.store(vs, L::VS);
    }
    float qf[KQ];
    float den = 0.f;                                           // q . n_0, this lane group's share
    {
        const float* qr = p + (int64_t)min(i, n - 1) * stride + (int64_t)head * dk;
        const float* n0 = N0 + at * dk;
#pragma unroll
        for (int s = 0; s < KQ; ++s) {
            const int kk = 4 * s + g;
            const float x = qr[min(kk, dk - 1)], y = n0[min(kk, dk - 1)];
            qf[s] = row_ok && kk < dk ? x * q_scale : 0.f;
            den = fmaf(qf[s], kk < dk ? y : 0.f, den);
        }
    }
    // the start state's first 64 key channels, on their way during the scores
    const float* s0 = S0 + at * dk * dv;
    Tile<4 * NV> ts;
    ts.template load<VEC>(s0, dv, min(dk, 64), 0, dv);
    __syncthreads();
    const double Mi = sM[i];
    const float carried = expf((float)((double)m0 - Mi));
    den *= carried;
    // scores against the keys of this row's past in the chunk, weighted
    floatx4 st[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        st[t] = floatx4{0.f, 0.f, 0.f, 0.f};
        if (t > wave || 16 * t >= n) continue;                 // uniform over the wave
#pragma unroll
        for (int s = 0; s < KQ; ++s)
            st[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(16 * t + r16) * L::KS + 4 * s + g], qf[s], st[t], 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int j = 16 * t + 4 * g + r;
            st[t][r] = j <= i ? st[t][r] * expf((float)(sc[j] - Mi)) : 0.f;
            den += st[t][r];
        }
    }
    den = rows4_sum(den);
    const float inv = 1.f / (fmaxf(fabsf(den), expf(-sm[i])) + 1e-6f);
    floatx4 o[NV];
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) o[vt] = floatx4{0.f, 0.f, 0.f, 0.f};
    // what the chunk's start state gives: o = S_0^T q, then times the row's factor
#pragma unroll
    for (int b = 0; b < (KQ + 15) / 16; ++b) {
        if (64 * b >= dk) continue;
        __syncthreads();                                       // the keys (or the channels before) have been read
        ts.store(ks, L::SS);
        __syncthreads();
        if (64 * (b + 1) < dk) ts.template load<VEC>(s0 + (int64_t)64 * (b + 1) * dv, dv, min(dk - 64 * (b + 1), 64), 0, dv);
#pragma unroll
        for (int s = 0; s < (KQ < 16 ? KQ : 16); ++s) {
            const float* sr = ks + (4 * s + g) * L::SS + r16;
#pragma unroll
            for (int vt = 0; vt < NV; ++vt)
                o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sr[16 * vt], qf[(16 * b + s) % KQ], o[vt], 0, 0, 0);
        }
    }
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) o[vt] *= carried;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        if (t > wave || 16 * t >= n) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float* vr = vs + (16 * t + 4 * g + r) * L::VS + r16;
#pragma unroll
            for (int vt = 0; vt < NV; ++vt)
                o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(vr[16 * vt], st[t][r], o[vt], 0, 0, 0);
        }
    }
    // o[vt][r]: value channel 16 vt + 4 g + r of row i
    float ss = 0.f;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            o[vt][r] *= inv;
            ss = fmaf(o[vt][r], o[vt][r], ss);                 // (channels past dv are zeros)
        }
    ss = rows4_sum(ss);
    if (!row_ok) return;
    const float rms = 1.f / sqrtf(ss / (float)dv + eps);
    const float* gate = p + (int64_t)i * stride + sh.g_off() + (int64_t)head * dv;
    const float* gn = gain + (int64_t)head * dv;
    T* dst = out + (row0 + i) * ((int64_t)sh.heads * dv) + (int64_t)head * dv;
    const bool whole = (dv & 3) == 0;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
        const int v0 = 16 * vt + 4 * g;
        if (v0 >= dv) continue;
        const float4 z = load_piece<VEC>(gate, v0, dv, true), w = load_piece<VEC>(gn, v0, dv, true);
        const float y[4] = {o[vt][0] * rms * w.x / (1.f + expf(-z.x)), o[vt][1] * rms * w.y / (1.f + expf(-z.y)),
                            o[vt][2] * rms * w.z / (1.f + expf(-z.z)), o[vt][3] * rms * w.w / (1.f + expf(-z.w))};
        if (whole) Elem<T>::store4(dst + v0, y);
        else
            for (int r = 0; r < 4 && v0 + r < dv; ++r) Elem<T>::store(dst + v0 + r, y[r]);
    }
}

}  // namespace st

using namespace st;

static int memory_check(const MemoryShape& sh, int64_t stride, int64_t slot_stride, float cap, float eps) {
    ST_CHECK(sh.heads > 0 && sh.dk > 0 && sh.dv > 0, "matrix_memory: bad sizes");
    ST_CHECK(sh.dk <= kMemMaxDim && sh.dv <= kMemMaxDim, "matrix_memory: up to %d key and value channels a head, not %d and %d",
             kMemMaxDim, sh.dk, sh.dv);
    ST_CHECK(stride >= sh.row(), "matrix_memory: rows of %lld floats are shorter than q, k, v, the gate and the log gates (%lld)",
             (long long)stride, (long long)sh.row());
    ST_CHECK(slot_stride >= sh.slot(), "matrix_memory: a slot of %lld floats is smaller than the state (%lld)",
             (long long)slot_stride, (long long)sh.slot());
    ST_CHECK(cap > 0.f && eps > 0.f, "matrix_memory: the gates' cap and eps must be positive");
    return 0;
}

// Kernels with more LDS than a launch may ask for by default have their limit raised, once each.
static int raise_lds(const void* kernel, size_t bytes) {
    static std::mutex mutex;
    static std::set<const void*> raised;
    if (bytes <= 48 * 1024) return 0;
    std::lock_guard<std::mutex> lock(mutex);
    if (raised.count(kernel)) return 0;
    ST_CHECK(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) == hipSuccess,
             "memory_chunks: cannot raise the LDS limit to %zu bytes", bytes);
    raised.insert(kernel);
    return 0;
}

// Every item has one row.
extern "C" int st_memory_step(void* out, const float* proj, int64_t stride, float* state, int64_t slot_stride,
                              const float* bias_i, const float* bias_f, const float* gain, const int* item_len,
                              const int* item_tok_off, const int* item_slot, int num_items, int heads, int key_dim,
                              int value_dim, float cap, float q_scale, float eps, int dtype, hipStream_t stream) {
    const MemoryShape sh{heads, key_dim, value_dim};
    if (memory_check(sh, stride, slot_stride, cap, eps)) return 1;
    ST_CHECK(num_items >= 0 && num_items <= 65535, "memory_step: %d items", num_items);
    if (num_items == 0) return 0;
    ST_CHECK(out && proj && state && bias_i && bias_f && gain && item_len && item_tok_off && item_slot,
             "memory_step: null operand");
    const bool vec = value_dim % 4 == 0 && slot_stride % 4 == 0 && ((uintptr_t)state & 15) == 0;
    const int cols = value_dim / (vec ? 4 : 1);
    const int pieces = cols * key_dim;
    int threads = 256;
    while (threads < 1024 && threads < pieces) threads <<= 1;
    const int lanes = threads / cols < key_dim ? threads / cols : key_dim;       // (cols <= 256 <= threads)
    const size_t lds = sizeof(float) * ((size_t)2 * key_dim + (size_t)lanes * value_dim + 16);
    ST_CHECK(lds <= 64 * 1024, "memory_step: %zu bytes of LDS", lds);
    const dim3 grid(heads, num_items);
#define ST_MS(T, V)                                                                                                     \
    memory_step_kernel<T, V><<<grid, threads, lds, stream>>>((T*)out, proj, stride, state, slot_stride, bias_i, bias_f, gain, \
        item_len, item_tok_off, item_slot, sh, cap, q_scale, eps, lanes)
    if (dtype == kF32) { if (vec) ST_MS(float, 4); else ST_MS(float, 1); }
    else if (dtype == kBF16) { if (vec) ST_MS(bf16_t, 4); else ST_MS(bf16_t, 1); }
    else ST_CHECK(false, "memory_step: unknown dtype %d", dtype);
#undef ST_MS
    ST_LAUNCH_CHECK("memory_step");
    return 0;
}

extern "C" int st_memory_chunk_rows() { return kMemChunk; }

// scratch_u [chunks, heads, dk, dv], scratch_n [chunks, heads, dk], scratch_s doubles [chunks, heads, 2], scratch_m
// [chunks, heads]; chunks >= num_rows / 64 + num_items.
extern "C" int st_memory_chunks(void* out, const float* proj, int64_t stride, float* state, int64_t slot_stride,
                                const float* bias_i, const float* bias_f, const float* gain, const int* item_len,
                                const int* item_tok_off, const int* item_slot, int num_items, int num_rows, int heads,
                                int key_dim, int value_dim, float cap, float q_scale, float eps, float* scratch_u,
                                float* scratch_n, double* scratch_s, float* scratch_m, int64_t scratch_chunks, int dtype,
                                hipStream_t stream) {
    const MemoryShape sh{heads, key_dim, value_dim};
    if (memory_check(sh, stride, slot_stride, cap, eps)) return 1;
    ST_CHECK(num_items >= 0 && num_rows >= 0, "memory_chunks: bad sizes");
    if (num_items == 0 || num_rows == 0) return 0;
    ST_CHECK(out && proj && state && bias_i && bias_f && gain && item_len && item_tok_off && item_slot && scratch_u &&
             scratch_n && scratch_s && scratch_m, "memory_chunks: null operand");
    ST_CHECK(dtype == kF32 || dtype == kBF16, "memory_chunks: unknown dtype %d", dtype);
    const int64_t chunks = num_rows / kMemChunk + num_items;   // every item's last chunk may be a short one
    ST_CHECK(scratch_chunks >= chunks, "memory_chunks: scratch for %lld chunks, %lld needed", (long long)scratch_chunks,
             (long long)chunks);
    ST_CHECK(chunks <= 65535 && num_items <= 65535, "memory_chunks: too many chunks or items");
    // 16-byte loads where every section of a row and every row of the state starts on a 16-byte border
    const bool vec = key_dim % 4 == 0 && value_dim % 4 == 0 && stride % 4 == 0 &&
                     (((uintptr_t)proj | (uintptr_t)scratch_u | (uintptr_t)gain) & 15) == 0;
    const dim3 grid1(heads, (unsigned)chunks, (value_dim + 63) / 64);
#define ST_MS2(KQ, VEC)                                                                                                \
    do {                                                                                                               \
        auto kernel = memory_sums_kernel<KQ, VEC>;                                                                      \
        const size_t lds = sizeof(float) * (size_t)(kMemChunk * (4 * KQ + 4) + kMemChunk * 68 + kMemChunk);              \
        if (raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;                                            \
        kernel<<<grid1, 256, lds, stream>>>(scratch_u, scratch_n, scratch_s, proj, stride, bias_i, bias_f, item_len,     \
                                            item_tok_off, item_slot, num_items, sh, cap);                               \
    } while (0)
#define ST_MS1(KQ) do { if (vec) ST_MS2(KQ, true); else ST_MS2(KQ, false); } while (0)
    if (key_dim <= 16) ST_MS1(4);
    else if (key_dim <= 32) ST_MS1(8);
    else if (key_dim <= 64) ST_MS1(16);
    else if (key_dim <= 128) ST_MS1(32);
    else ST_MS1(64);
#undef ST_MS1
#undef ST_MS2
    ST_LAUNCH_CHECK("memory_chunks (sums)");
    const int elements = key_dim * value_dim + key_dim;
    memory_carry_kernel<<<dim3(heads, num_items, (elements + 255) / 256), 256, 0, stream>>>(
        scratch_u, scratch_n, scratch_s, scratch_m, state, slot_stride, item_len, item_slot, sh);
    ST_LAUNCH_CHECK("memory_chunks (carry)");
    const dim3 grid(heads, (unsigned)chunks);
#define ST_MO_E(T, KQ, NV, VEC)                                                                                        \
    do {                                                                                                               \
        auto kernel = memory_out_kernel<T, KQ, NV, VEC>;                                                                \
        constexpr size_t lds = MemoryOutLds<KQ, NV>::bytes;                                                             \
        if (raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;                                            \
        kernel<<<grid, 256, lds, stream>>>((T*)out, proj, stride, state, slot_stride, scratch_u, scratch_n, scratch_m, bias_i, \
            bias_f, gain, item_len, item_tok_off, item_slot, num_items, sh, cap, q_scale, eps);                         \
    } while (0)
#define ST_MO(T, KQ, NV) do { if (vec) ST_MO_E(T, KQ, NV, true); else ST_MO_E(T, KQ, NV, false); } while (0)
#define ST_MO_V(T, KQ) do { if (value_dim <= 64) ST_MO(T, KQ, 4); else if (value_dim <= 128) ST_MO(T, KQ, 8); else ST_MO(T, KQ, 16); } while (0)
#define ST_MO_K(T) do { if (key_dim <= 16) ST_MO_V(T, 4); else if (key_dim <= 32) ST_MO_V(T, 8); else if (key_dim <= 64) ST_MO_V(T, 16); \
                        else if (key_dim <= 128) ST_MO_V(T, 32); else ST_MO_V(T, 64); } while (0)
    if (dtype == kF32) ST_MO_K(float); else ST_MO_K(bf16_t);
#undef ST_MO_K
#undef ST_MO_V
#undef ST_MO
#undef ST_MO_E
    ST_LAUNCH_CHECK("memory_chunks (outputs)");
    return 0;
}
