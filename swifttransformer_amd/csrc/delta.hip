// Gated delta rule, for batches of portions of sequences.  A head keeps a float matrix S [key channels x value channels];
// per token, after a short causal filter a channel with SiLU on q, k and v, q and k brought to unit length and q scaled,
//
//   g = exp(-exp(a_log) softplus(za + dt_bias));   b = sigmoid(zb)                       one of each a head
//   S <- g S;   u = b (v - S^T k);   S <- S + k u^T;   o = S^T q
//   y = o / sqrt(mean(o^2) + eps) * gain * silu(z)                                       per head, gain shared by heads
//
// Heads share q and k in groups of neighbours.  Two routes over one state.  A step of single tokens is one kernel
// (`step`), a workgroup a head and request: filter, unit vectors, gates, state, read-out, norm and gate.  Other steps:
// `inputs` (filter, unit vectors, gates, all rows side by side), then chunks of 64 rows, counted from an item's first row
// of the step.  With G_i the sum of log g over a chunk's rows up to i (double: the sums cancel in the exponents) and S_0
// the state at the chunk's start, the u of a chunk solve a unit triangular system,
//
//   u_i + sum_(j < i) A_ij u_j = b_i v_i - b_i e^(G_i) S_0^T k_i,     A_ij = b_i e^(G_i - G_j) (k_i . k_j),
//
// so U = W_v - W_k S_0 with W_v = (I + A)^-1 diag(b) V and W_k = (I + A)^-1 diag(b e^G) K, which need no state (`prep`,
// chunks side by side); `carry` walks a request's chunks, S <- e^(G_n) S + sum_j e^(G_n - G_j) k_j u_j^T, and leaves every
// chunk's U and start state; `outputs` forms o_i = e^(G_i) S_0^T q_i + sum_(j <= i) e^(G_i - G_j) (q_i . k_j) u_j with norm
// and gate.  No exponent is positive.  All products are float on the matrix cores (v_mfma_f32_16x16x4_f32).
//
// A row of `proj` is q | k | v | z | zb | za: (qk heads x dk) twice, (heads x dv) twice, heads twice, floats.
// A slot is a ring of the filter's inputs [taps, channels] (q | k | v; position p at p % taps: a single token's entry is
// none of those that its filter reads) | S [heads, dk, dv], at a multiple of 4 floats.
#include "api.h"
#include "chunk_tiles.h"
#include "common.h"

#include <mutex>
#include <set>

namespace st {

typedef float floatx4 __attribute__((ext_vector_type(4)));

constexpr int kDeltaMaxDim = 256, kDeltaMaxTaps = 8;

struct DeltaShape {
    int heads, qk_heads, dk, dv, taps;
    __host__ __device__ int64_t k_off() const { return (int64_t)qk_heads * dk; }
    __host__ __device__ int64_t v_off() const { return 2 * k_off(); }
    __host__ __device__ int64_t channels() const { return v_off() + (int64_t)heads * dv; }
    __host__ __device__ int64_t z_off() const { return channels(); }
    __host__ __device__ int64_t b_off() const { return z_off() + (int64_t)heads * dv; }
    __host__ __device__ int64_t a_off() const { return b_off() + heads; }
    __host__ __device__ int64_t row() const { return a_off() + heads; }
    __host__ __device__ int64_t s_base() const { return (taps * channels() + 3) / 4 * 4; }
    __host__ __device__ int64_t slot() const { return s_base() + (int64_t)heads * dk * dv; }
};

__device__ inline float delta_silu(float x) { return x / (1.f + expf(-x)); }
__device__ inline float delta_log_decay(float z, float a_log, float dt_bias) {
    const float x = z + dt_bias;
    return -expf(a_log) * (x > 20.f ? x : log1pf(expf(x)));
}

// sums of three numbers over a workgroup; red: 48 floats
__device__ inline void block_sum3(float& a, float& b, float& c, float* red) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
    a = wave_sum(a); b = wave_sum(b); c = wave_sum(c);
    __syncthreads();
    if (lane == 0) { red[wave] = a; red[16 + wave] = b; red[32 + wave] = c; }
    __syncthreads();
    a = b = c = 0.f;
    for (int w = 0; w < waves; ++w) { a += red[w]; b += red[16 + w]; c += red[32 + w]; }
}

// ---------------------------------------------------------------- single tokens
// A workgroup a (head, item).  A thread owns V neighbouring value channels of every `lanes`-th key channel, NP of them in
// registers.  LDS: q | k | v after the filter [2 dk + dv] | u [dv] | partial sums S^T k, S^T q [2][lanes][dv] | red [48].
template <typename T, int V, int NP>
__global__ __launch_bounds__(1024) void delta_step_kernel(
    T* __restrict__ out, const float* __restrict__ proj, int64_t stride, float* __restrict__ state, int64_t slot_stride,
    const float* __restrict__ taps_w, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    const float* __restrict__ gain, const int* __restrict__ positions, const int* __restrict__ item_len,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, DeltaShape sh, float q_scale, float unit_eps,
    float eps, int lanes) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int head = blockIdx.x, item = blockIdx.y, tid = threadIdx.x;
    const int slot = item_slot[item];
    if (slot < 0 || item_len[item] <= 0) return;
    const int64_t row = item_tok_off[item];
    const int dk = sh.dk, dv = sh.dv, taps = sh.taps, cols = dv / V, rep = sh.heads / sh.qk_heads, group = head / rep;
    const int64_t C = sh.channels();
    const float* p = proj + row * stride;
    float* ring = state + (int64_t)slot * slot_stride;
    float* S = ring + sh.s_base() + (int64_t)head * dk * dv;
    float* sx = lds;
    float* su = sx + 2 * dk + dv;
    float* part = su + dv;
    float* red = part + 2 * lanes * dv;
    const int pos = positions[row];
    const int c = tid % cols, kl = tid / cols;
    const bool works = kl < lanes;
    float s[NP][V];
    if (works) {
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const float* src = S + (int64_t)min(i * lanes + kl, dk - 1) * dv + c * V;
            if (V == 4) {
                const float4 x = *reinterpret_cast<const float4*>(src);
                s[i][0] = x.x; s[i][1 % V] = x.y; s[i][2 % V] = x.z; s[i][3 % V] = x.w;
            } else {
                s[i][0] = src[0];
            }
        }
    }
    const float zb = p[sh.b_off() + head], za = p[sh.a_off() + head];
    for (int e = tid; e < 2 * dk + dv; e += blockDim.x) {
        const int64_t ch = e < dk ? (int64_t)group * dk + e
                         : e < 2 * dk ? sh.k_off() + (int64_t)group * dk + (e - dk) : sh.v_off() + (int64_t)head * dv + (e - 2 * dk);
        const float x0 = p[ch];
        float back[kDeltaMaxTaps];
#pragma unroll
        for (int j = 1; j < kDeltaMaxTaps; ++j) back[j] = j < taps && pos >= j ? ring[(int64_t)((pos - j) % taps) * C + ch] : 0.f;
        float acc = taps_w[(int64_t)(taps - 1) * C + ch] * x0;
#pragma unroll
        for (int j = 1; j < kDeltaMaxTaps; ++j)
            if (j < taps) acc = fmaf(taps_w[(int64_t)(taps - 1 - j) * C + ch], back[j], acc);
        if (e >= 2 * dk || head % rep == 0) ring[(int64_t)(pos % taps) * C + ch] = x0;
        sx[e] = delta_silu(acc);
    }
    const float strength = 1.f / (1.f + expf(-zb)), decay = expf(delta_log_decay(za, a_log[head], dt_bias[head]));
    __syncthreads();
    float qq = 0.f, kk2 = 0.f, qk = 0.f;
    if (tid < dk) { const float a = sx[tid], b = sx[dk + tid]; qq = a * a; kk2 = b * b; qk = a * b; }
    block_sum3(qq, kk2, qk, red);
    const float fq = q_scale / sqrtf(qq + unit_eps), fk = 1.f / sqrtf(kk2 + unit_eps);
    qk *= fq * fk;
    if (works) {
        float rk[V], rq[V];
#pragma unroll
        for (int e = 0; e < V; ++e) rk[e] = rq[e] = 0.f;
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int kk = i * lanes + kl;
            if (kk >= dk) continue;
            const float a = sx[kk], b = sx[dk + kk];
#pragma unroll
            for (int e = 0; e < V; ++e) { rk[e] = fmaf(s[i][e], b, rk[e]); rq[e] = fmaf(s[i][e], a, rq[e]); }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) {
            part[kl * dv + c * V + e] = rk[e];
            part[(lanes + kl) * dv + c * V + e] = rq[e];
        }
    }
    __syncthreads();
    float o = 0.f;
    if (tid < dv) {
        float rk = 0.f, rq = 0.f;
        for (int j = 0; j < lanes; ++j) { rk += part[j * dv + tid]; rq += part[(lanes + j) * dv + tid]; }
        const float u = strength * (sx[2 * dk + tid] - decay * (rk * fk));
        o = fmaf(decay, rq * fq, qk * u);
        su[tid] = u;
    }
    const float ss = block_sum(o * o, red);          // (its barriers also order u)
    if (works) {
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int kk = i * lanes + kl;
            if (kk >= dk) continue;
            const float kn = sx[dk + kk] * fk;
#pragma unroll
            for (int e = 0; e < V; ++e) s[i][e] = fmaf(decay, s[i][e], kn * su[c * V + e]);
            float* dst = S + (int64_t)kk * dv + c * V;
            if (V == 4) *reinterpret_cast<float4*>(dst) = make_float4(s[i][0], s[i][1 % V], s[i][2 % V], s[i][3 % V]);
            else dst[0] = s[i][0];
        }
    }
    if (tid < dv) {
        const float y = o / sqrtf(ss / (float)dv + eps) * gain[tid] * delta_silu(p[sh.z_off() + (int64_t)head * dv + tid]);
        Elem<T>::store(out + row * ((int64_t)sh.heads * dv) + (int64_t)head * dv + tid, y);
    }
}

// ---------------------------------------------------------------- rows side by side
// qkv [rows, channels]: the filter with SiLU, q and k at unit length (q scaled); gates [rows, 2 heads]: strength | log decay.
// A wave takes 8 consecutive rows of one unit: as many q and k heads as have whole segments of 64 channels in four, 256 value
// channels, or the gates; the filter's inputs of a row's past are the rows above in its item, before those the ring.  TM:
// taps at most; SEG: segments of a head (1, 2 or 4).
constexpr int kInputRows = 8;
__host__ __device__ inline int delta_head_units(const DeltaShape& sh, int seg) { return (2 * sh.qk_heads + 4 / seg - 1) / (4 / seg); }
template <int TM, int SEG>
__global__ __launch_bounds__(256) void delta_inputs_kernel(
    float* __restrict__ qkv, float* __restrict__ gates, const float* __restrict__ proj, int64_t stride,
    const float* __restrict__ state, int64_t slot_stride, const float* __restrict__ taps_w, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const int* __restrict__ token_item, const int* __restrict__ positions,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int num_tokens, int units, DeltaShape sh,
    float q_scale, float unit_eps) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6), t0 = blockIdx.x * kInputRows;
    if (unit >= units) return;
    const int64_t C = sh.channels();
    if (unit == units - 1) {                         // the gates
        for (int e = lane; e < kInputRows * sh.heads; e += 64) {
            const int t = t0 + e / sh.heads, h = e % sh.heads;
            if (t >= num_tokens) continue;
            const float* p = proj + (int64_t)t * stride;
            gates[(int64_t)t * 2 * sh.heads + h] = 1.f / (1.f + expf(-p[sh.b_off() + h]));
            gates[(int64_t)t * 2 * sh.heads + sh.heads + h] = delta_log_decay(p[sh.a_off() + h], a_log[h], dt_bias[h]);
        }
        return;
    }
    const int head_units = delta_head_units(sh, SEG), taps = sh.taps;
    const bool unit_vector = unit < head_units;
    constexpr int L = 4;                             // channels a lane: segment e of 64
    int64_t ch[L];
    bool ok[L];
    float factor[L];
#pragma unroll
    for (int e = 0; e < L; ++e) {
        if (unit_vector) {
            const int head = unit * (L / SEG) + e / SEG, c = (e % SEG) * 64 + lane;
            ok[e] = head < 2 * sh.qk_heads && c < sh.dk;
            ch[e] = ok[e] ? (int64_t)head * sh.dk + c : 0;
            factor[e] = head < sh.qk_heads ? q_scale : 1.f;
        } else {
            const int64_t c = sh.v_off() + (int64_t)(unit - head_units) * 256 + 64 * e + lane;
            ok[e] = c < C;
            ch[e] = ok[e] ? c : 0;
            factor[e] = 1.f;
        }
    }
    float x[kInputRows + TM - 1][L], w[TM][L];
#pragma unroll
    for (int i = 0; i < kInputRows + TM - 1; ++i) {
        const int t = min(max(t0 + i - (TM - 1), 0), num_tokens - 1);
#pragma unroll
        for (int e = 0; e < L; ++e) x[i][e] = proj[(int64_t)t * stride + ch[e]];
    }
#pragma unroll
    for (int j = 0; j < TM; ++j)
#pragma unroll
        for (int e = 0; e < L; ++e) w[j][e] = j < taps ? taps_w[(int64_t)(taps - 1 - j) * C + ch[e]] : 0.f;
#pragma unroll
    for (int r = 0; r < kInputRows; ++r) {
        const int t = t0 + r;
        if (t >= num_tokens) return;
        const int item = token_item[t];
        if (item < 0) continue;                      // a padding row
        const int in_item = t - item_tok_off[item], pos = positions[t];
        const float* ring = state + (int64_t)item_slot[item] * slot_stride;
        float acc[L];
#pragma unroll
        for (int e = 0; e < L; ++e) acc[e] = w[0][e] * x[r + TM - 1][e];
#pragma unroll
        for (int j = 1; j < TM; ++j) {
            if (j >= taps) continue;
            if (in_item >= j) {
#pragma unroll
                for (int e = 0; e < L; ++e) acc[e] = fmaf(w[j][e], x[r + TM - 1 - j][e], acc[e]);
            } else if (pos >= j) {
#pragma unroll
                for (int e = 0; e < L; ++e)
                    acc[e] = fmaf(w[j][e], ring[(int64_t)((pos - j) % taps) * C + ch[e]], acc[e]);
            }
        }
#pragma unroll
        for (int e = 0; e < L; ++e) acc[e] = ok[e] ? delta_silu(acc[e]) : 0.f;
        if (unit_vector) {
#pragma unroll
            for (int h = 0; h < L / SEG; ++h) {
                float ss = 0.f;
#pragma unroll
                for (int e = h * SEG; e < (h + 1) * SEG; ++e) ss = fmaf(acc[e], acc[e], ss);
                const float f = 1.f / sqrtf(wave_sum(ss) + unit_eps);
#pragma unroll
                for (int e = h * SEG; e < (h + 1) * SEG; ++e) acc[e] *= f * factor[e];
            }
        }
#pragma unroll
        for (int e = 0; e < L; ++e)
            if (ok[e]) qkv[(int64_t)t * C + ch[e]] = acc[e];
    }
}

// ---------------------------------------------------------------- chunks
// The first wave: G_i (inclusive sums of the log decays) of a chunk's n rows; past them the last one's.
__device__ inline double delta_chunk_decay(const float* __restrict__ log_decay, int64_t stride, int n) {
    const int lane = threadIdx.x & 63;
    double G = lane < n ? (double)log_decay[(int64_t)lane * stride] : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const double up = __shfl_up(G, o, 64);
        if (lane >= o) G += up;
    }
    return G;
}

// What a chunk needs no state for.  Grid (heads, chunks).  wv [chunk, head, 64, dv] and wk [.., 64, dk]: the triangular
// system solved for its two right sides, a thread a column; kt [.., dk, 64]: e^(G_n - G_j) k_j, transposed; fall [chunk,
// head]: e^(G_n).  KQ: dk <= 4 KQ.  LDS: G doubles [64] | b [64] | k [64][4 KQ + 4] | A [64][68].
template <int KQ, bool VEC>
__global__ __launch_bounds__(256) void delta_prep_kernel(
    float* __restrict__ wv, float* __restrict__ wk, float* __restrict__ kt, float* __restrict__ fall,
    const float* __restrict__ qkv, const float* __restrict__ gates, const int* __restrict__ item_len,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int num_items, DeltaShape sh) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int head = blockIdx.x, idx = blockIdx.y, tid = threadIdx.x;
    int item, chunk;
    if (!find_chunk(idx, item_len, item_slot, num_items, item, chunk)) return;
    constexpr int KS = 4 * KQ + 4, AS = kChunkRows + 4;
    const int n = min(kChunkRows, item_len[item] - chunk * kChunkRows);
    const int64_t row0 = (int64_t)item_tok_off[item] + (int64_t)chunk * kChunkRows, C = sh.channels();
    const int dk = sh.dk, dv = sh.dv, group = head / (sh.heads / sh.qk_heads);
    double* sG = reinterpret_cast<double*>(lds);
    float* sb = reinterpret_cast<float*>(sG + kChunkRows);
    float* ks = sb + kChunkRows;
    float* sa = ks + kChunkRows * KS;
    const float* base = qkv + row0 * C;
    const float* gt = gates + row0 * 2 * sh.heads;
    Tile<KQ> tk;
    tk.template load<VEC>(base + sh.k_off() + (int64_t)group * dk, C, n, 0, dk);
    if (tid < 64) {
        sG[tid] = delta_chunk_decay(gt + sh.heads + head, 2 * sh.heads, n);
        sb[tid] = tid < n ? gt[(int64_t)tid * 2 * sh.heads + head] : 0.f;
    }
    tk.store(ks, KS);
    __syncthreads();
    const int lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    // A by 16 x 16 tiles on and below the diagonal
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        if (t > wave) continue;                      // uniform over the wave
        floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KQ; ++s)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(16 * wave + r16) * KS + 4 * s + g], ks[(16 * t + r16) * KS + 4 * s + g], acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = 16 * wave + 4 * g + r, j = 16 * t + r16;
            sa[i * AS + j] = j < i && i < n ? sb[i] * expf((float)(sG[i] - sG[j])) * acc[r] : 0.f;
        }
    }
    const int64_t at = (int64_t)idx * sh.heads + head;
    const double last = sG[kChunkRows - 1];
    if (tid == 0) fall[at] = expf((float)last);
    for (int e = tid; e < dk * kChunkRows; e += 256) {
        const int c = e / kChunkRows, j = e % kChunkRows;
        kt[at * dk * kChunkRows + e] = expf((float)(last - sG[j])) * ks[j * KS + c];
    }
    __syncthreads();
    for (int c = tid; c < dv + dk; c += 256) {
        float x[kChunkRows];
        const bool is_v = c < dv;
        if (is_v) {
            const float* vp = base + sh.v_off() + (int64_t)head * dv + c;
#pragma unroll
            for (int i = 0; i < kChunkRows; ++i) x[i] = vp[(int64_t)min(i, n - 1) * C];
#pragma unroll
            for (int i = 0; i < kChunkRows; ++i) x[i] *= sb[i];        // (no strength past the chunk's rows)
        } else {
#pragma unroll
            for (int i = 0; i < kChunkRows; ++i) x[i] = sb[i] * expf((float)sG[i]) * ks[i * KS + c - dv];
        }
#pragma unroll
        for (int i = 1; i < kChunkRows; ++i) {
            float acc = x[i];
#pragma unroll
            for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
                const float4 a = *reinterpret_cast<const float4*>(sa + i * AS + 4 * j4);   // (zeros from the diagonal on)
                acc = fmaf(-a.x, x[4 * j4], acc);
                if (4 * j4 + 1 < i) acc = fmaf(-a.y, x[4 * j4 + 1], acc);
                if (4 * j4 + 2 < i) acc = fmaf(-a.z, x[4 * j4 + 2], acc);
                if (4 * j4 + 3 < i) acc = fmaf(-a.w, x[4 * j4 + 3], acc);
            }
            x[i] = acc;
        }
        float* dst = is_v ? wv + at * kChunkRows * dv + c : wk + at * kChunkRows * dk + (c - dv);
        const int step = is_v ? dv : dk;
#pragma unroll
        for (int i = 0; i < kChunkRows; ++i) dst[(int64_t)i * step] = x[i];
    }
}

// Grid (heads, blocks of 16 value channels, items): walks a request's chunks.  wv becomes U, start [chunk, head, dk, dv]
// receives the chunks' start states.  A wave owns 16 rows of U and every fourth tile of 16 key channels of S; both meet in
// LDS: S [16 KT][20] | U [64][20].  The matrix instruction's four depth slots are key channels (rows) 4 g + r, so that the
// results of one product are the operands of the next as they lie.  KT: dk <= 16 KT; AHEAD: chunks whose operands are on
// their way at a time (a trip to memory takes longer than a chunk).
template <int KT, int AHEAD>
__global__ __launch_bounds__(256) void delta_carry_kernel(
    float* __restrict__ wv, const float* __restrict__ wk, const float* __restrict__ kt, const float* __restrict__ fall,
    float* __restrict__ start, float* __restrict__ state, int64_t slot_stride, const int* __restrict__ item_len,
    const int* __restrict__ item_slot, DeltaShape sh) {
    __shared__ float ss[16 * KT][20];
    __shared__ float su[kChunkRows][20];
    const int head = blockIdx.x, vb = blockIdx.y * 16, item = blockIdx.z, tid = threadIdx.x;
    const int slot = item_slot[item], len = item_len[item];
    if (slot < 0 || len <= 0) return;
    int first = 0;
    for (int b = 0; b < item; ++b) {
        const int l = item_len[b];
        first += (item_slot[b] >= 0 && l > 0) ? (l + kChunkRows - 1) / kChunkRows : 0;
    }
    const int chunks = (len + kChunkRows - 1) / kChunkRows, dk = sh.dk, dv = sh.dv;
    const int lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4, col = vb + r16, colc = min(col, dv - 1);
    constexpr int MT = (KT + 3) / 4;                 // a wave's tiles of S
    float* home = state + (int64_t)slot * slot_stride + sh.s_base() + (int64_t)head * dk * dv;
    floatx4 S[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int kk = 16 * (wave + 4 * m) + 4 * g + r;
            const float v = home[(int64_t)min(kk, dk - 1) * dv + colc];
            S[m][r] = kk < dk && col < dv ? v : 0.f;
            if (wave + 4 * m < KT) ss[kk][r16] = S[m][r];
        }
    const bool quads = dk % 4 == 0;
    struct Operands {
        floatx4 fk[KT], ft[MT][4], fv;
    };
    auto load = [&](Operands& p, int c) {
        const int64_t at = (int64_t)(first + c) * sh.heads + head;
        const float* a = wk + (at * kChunkRows + 16 * wave + r16) * dk;
#pragma unroll
        for (int t = 0; t < KT; ++t) {
            const int kk = 16 * t + 4 * g;
            if (quads) {
                const float4 v = *reinterpret_cast<const float4*>(a + min(kk, dk - 4));
                p.fk[t] = kk < dk ? floatx4{v.x, v.y, v.z, v.w} : floatx4{0.f, 0.f, 0.f, 0.f};
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r) { const float v = a[min(kk + r, dk - 1)]; p.fk[t][r] = kk + r < dk ? v : 0.f; }
            }
        }
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            const int kk = 16 * (wave + 4 * m) + r16;
            const float* b = kt + (at * dk + min(kk, dk - 1)) * kChunkRows;
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                const float4 v = *reinterpret_cast<const float4*>(b + 16 * s + 4 * g);
                p.ft[m][s] = floatx4{v.x, v.y, v.z, v.w};     // (rows of channels past dk give rows of S that are not kept)
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) p.fv[r] = wv[(at * kChunkRows + 16 * wave + 4 * g + r) * dv + colc];
    };
    // (a lane holds the factor of chunk lane of the present 64: a load that is the same for all lanes would be a scalar one,
    // and every barrier waits for those)
    float falls = 0.f;
    auto step = [&](Operands& p, int c) {
        if ((c & 63) == 0) falls = fall[(int64_t)(first + min(c + lane, chunks - 1)) * sh.heads + head];
        const float keep = __shfl(falls, c & 63, 64);
        const int64_t at = (int64_t)(first + c) * sh.heads + head;
        floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < KT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(p.fk[t][r], ss[16 * t + 4 * g + r][r16], acc, 0, 0, 0);
        const floatx4 u = p.fv - acc;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            su[16 * wave + 4 * g + r][r16] = u[r];
            if (col < dv) wv[(at * kChunkRows + 16 * wave + 4 * g + r) * dv + col] = u[r];
        }
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int kk = 16 * (wave + 4 * m) + 4 * g + r;
                if (kk < dk && col < dv) start[(at * dk + kk) * dv + col] = S[m][r];
            }
        __syncthreads();                             // U is there, S has been read
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            if (wave + 4 * m >= KT) continue;
            floatx4 d = S[m] * keep;
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int r = 0; r < 4; ++r) d = __builtin_amdgcn_mfma_f32_16x16x4f32(p.ft[m][s][r], su[16 * s + 4 * g + r][r16], d, 0, 0, 0);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int kk = 16 * (wave + 4 * m) + 4 * g + r;
                S[m][r] = kk < dk ? d[r] : 0.f;
                ss[kk][r16] = S[m][r];
            }
        }
        if (c + AHEAD < chunks) load(p, c + AHEAD);
        __syncthreads();
    };
    Operands ops[AHEAD];
#pragma unroll
    for (int b = 0; b < AHEAD; ++b) load(ops[b], min(b, chunks - 1));
    __syncthreads();
    for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
#pragma unroll
        for (int b = 0; b < AHEAD; ++b)
            if (c0 + b < chunks) step(ops[b], c0 + b);       // uniform
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int kk = 16 * (wave + 4 * m) + 4 * g + r;
            if (kk < dk && col < dv) home[(int64_t)kk * dv + col] = S[m][r];
        }
}

// Rows of a chunk, transposed: S^T = K Q^T leaves a lane with keys 4 g + r of ONE row (lane % 16), so weights and the norm
// are per-lane numbers and sums over the four lane groups, and the weighted scores are the next product's operand as they
// lie.  Four waves, 16 rows each.  NV: dv <= 16 NV; KQ: dk <= 4 KQ.  LDS: G doubles [64] | k [64][4 KQ + 4], later 64 key
// channels of the start state [64][16 NV + 16] | U [64][16 NV + 4].  An item's last chunk also moves its ring on.
template <int KQ, int NV>
struct DeltaOutLds {
    static constexpr int KS = 4 * KQ + 4, VS = 16 * NV + 4, SS = 16 * NV + 16;
    static constexpr int first = KS > SS ? 64 * KS : 64 * SS;
    static constexpr size_t bytes = sizeof(double) * kChunkRows + sizeof(float) * (size_t)(first + 64 * VS);
};

template <typename T, int KQ, int NV, bool VEC>
__global__ __launch_bounds__(256) void delta_out_kernel(
    T* __restrict__ out, const float* __restrict__ proj, int64_t stride, const float* __restrict__ qkv,
    const float* __restrict__ gates, const float* __restrict__ U, const float* __restrict__ start, float* __restrict__ state,
    int64_t slot_stride, const float* __restrict__ gain, const int* __restrict__ positions, const int* __restrict__ item_len,
    const int* __restrict__ item_tok_off, const int* __restrict__ item_slot, int num_items, DeltaShape sh, float eps) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    using L = DeltaOutLds<KQ, NV>;
    const int head = blockIdx.x, idx = blockIdx.y, tid = threadIdx.x;
    int item, chunk;
    if (!find_chunk(idx, item_len, item_slot, num_items, item, chunk)) return;
    const int len = item_len[item], n = min(kChunkRows, len - chunk * kChunkRows);
    const int64_t row0 = (int64_t)item_tok_off[item] + (int64_t)chunk * kChunkRows, C = sh.channels();
    const int dk = sh.dk, dv = sh.dv, rep = sh.heads / sh.qk_heads, group = head / rep;
    double* sG = reinterpret_cast<double*>(lds);
    float* ks = reinterpret_cast<float*>(sG + kChunkRows);
    float* vs = ks + L::first;
    const int64_t at = (int64_t)idx * sh.heads + head;
    const int lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int i = wave * 16 + r16;                   // this lane's row of the chunk
    const bool row_ok = i < n;
    if ((chunk + 1) * kChunkRows >= len) {           // the filter's inputs of the item's last rows
        float* ring = state + (int64_t)item_slot[item] * slot_stride;
        const int m = min(len, sh.taps), e0 = head % rep == 0 ? 0 : 2 * dk;
        for (int e = e0 + tid; e < 2 * dk + dv; e += 256) {
            const int64_t ch = e < dk ? (int64_t)group * dk + e
                             : e < 2 * dk ? sh.k_off() + (int64_t)group * dk + (e - dk) : sh.v_off() + (int64_t)head * dv + (e - 2 * dk);
            for (int b = 0; b < m; ++b) {
                const int64_t t = (int64_t)item_tok_off[item] + len - m + b;
                ring[(int64_t)(positions[t] % sh.taps) * C + ch] = proj[t * stride + ch];
            }
        }
    }
    {
        Tile<KQ> tk;
        Tile<4 * NV> tv;
        tk.template load<VEC>(qkv + row0 * C + sh.k_off() + (int64_t)group * dk, C, n, 0, dk);
        tv.template load<VEC>(U + at * kChunkRows * dv, dv, n, 0, dv);
        if (tid < 64) sG[tid] = delta_chunk_decay(gates + row0 * 2 * sh.heads + sh.heads + head, 2 * sh.heads, n);
        tk.store(ks, L::KS);
        tv.store(vs, L::VS);
    }
    float qf[KQ];
    {
        const float* qr = qkv + (row0 + min(i, n - 1)) * C + (int64_t)group * dk;
#pragma unroll
        for (int s = 0; s < KQ; ++s) {
            const int kk = 4 * s + g;
            const float x = qr[min(kk, dk - 1)];
            qf[s] = row_ok && kk < dk ? x : 0.f;
        }
    }
    const float* s0 = start + at * dk * dv;
    Tile<4 * NV> ts;                                 // the start state's first 64 key channels, on their way during the scores
    ts.template load<VEC>(s0, dv, min(dk, 64), 0, dv);
    __syncthreads();
    const double Gi = sG[i];
    floatx4 st[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        st[t] = floatx4{0.f, 0.f, 0.f, 0.f};
        if (t > wave || 16 * t >= n) continue;       // uniform over the wave
#pragma unroll
        for (int s = 0; s < KQ; ++s)
            st[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(16 * t + r16) * L::KS + 4 * s + g], qf[s], st[t], 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int j = 16 * t + 4 * g + r;
            st[t][r] = j <= i ? st[t][r] * expf((float)(Gi - sG[j])) : 0.f;
        }
    }
    floatx4 o[NV];
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) o[vt] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < (KQ + 15) / 16; ++b) {       // S_0^T q, then times the row's factor
        if (64 * b >= dk) continue;
        __syncthreads();                             // the keys (or the channels before) have been read
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
    const float carried = expf((float)Gi);
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) o[vt] *= carried;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        if (t > wave || 16 * t >= n) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float* vr = vs + (16 * t + 4 * g + r) * L::VS + r16;
#pragma unroll
            for (int vt = 0; vt < NV; ++vt) o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(vr[16 * vt], st[t][r], o[vt], 0, 0, 0);
        }
    }
    // o[vt][r]: value channel 16 vt + 4 g + r of row i
    float ssum = 0.f;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt)
#pragma unroll
        for (int r = 0; r < 4; ++r) ssum = fmaf(o[vt][r], o[vt][r], ssum);
    ssum = rows4_sum(ssum);
    if (!row_ok) return;
    const float rms = 1.f / sqrtf(ssum / (float)dv + eps);
    const float* z = proj + (row0 + i) * stride + sh.z_off() + (int64_t)head * dv;
    T* dst = out + (row0 + i) * ((int64_t)sh.heads * dv) + (int64_t)head * dv;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
        const int v0 = 16 * vt + 4 * g;
        if (v0 >= dv) continue;
        const float4 zz = load_piece<VEC>(z, v0, dv, true), w = load_piece<VEC>(gain, v0, dv, true);
        const float y[4] = {o[vt][0] * rms * w.x * delta_silu(zz.x), o[vt][1] * rms * w.y * delta_silu(zz.y),
                            o[vt][2] * rms * w.z * delta_silu(zz.z), o[vt][3] * rms * w.w * delta_silu(zz.w)};
        if ((dv & 3) == 0) Elem<T>::store4(dst + v0, y);
        else
            for (int r = 0; r < 4 && v0 + r < dv; ++r) Elem<T>::store(dst + v0 + r, y[r]);
    }
}

}  // namespace st

using namespace st;

static int delta_check(const DeltaShape& sh, int64_t stride, int64_t slot_stride, float eps, float unit_eps) {
    ST_CHECK(sh.heads > 0 && sh.qk_heads > 0 && sh.heads % sh.qk_heads == 0 && sh.dk > 0 && sh.dv > 0, "delta_rule: bad sizes");
    ST_CHECK(sh.dk <= kDeltaMaxDim && sh.dv <= kDeltaMaxDim, "delta_rule: up to %d key and value channels a head, not %d and %d",
             kDeltaMaxDim, sh.dk, sh.dv);
    ST_CHECK(sh.taps >= 1 && sh.taps <= kDeltaMaxTaps, "delta_rule: 1 to %d taps, not %d", kDeltaMaxTaps, sh.taps);
    ST_CHECK(stride >= sh.row() && slot_stride >= sh.slot(), "delta_rule: rows of %lld floats and slots of %lld are too short",
             (long long)stride, (long long)slot_stride);
    ST_CHECK(eps > 0.f && unit_eps > 0.f, "delta_rule: eps must be positive");
    return 0;
}

// Kernels with more LDS than a launch may ask for by default have their limit raised, once each.
static int delta_raise_lds(const void* kernel, size_t bytes) {
    static std::mutex mutex;
    static std::set<const void*> raised;
    if (bytes <= 48 * 1024) return 0;
    std::lock_guard<std::mutex> lock(mutex);
    if (raised.count(kernel)) return 0;
    ST_CHECK(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) == hipSuccess,
             "delta_rule: cannot raise the LDS limit to %zu bytes", bytes);
    raised.insert(kernel);
    return 0;
}

extern "C" int64_t st_delta_slot(int heads, int qk_heads, int key_dim, int value_dim, int taps) {
    return DeltaShape{heads, qk_heads, key_dim, value_dim, taps}.slot();
}
extern "C" int st_delta_chunk_rows() { return kChunkRows; }

// Every item has one row.  taps_w [taps, channels]: the filters by tap, the last row the token's own.
extern "C" int st_delta_step(void* out, const float* proj, int64_t stride, float* state, int64_t slot_stride, const float* taps_w,
                             const float* a_log, const float* dt_bias, const float* gain, const int* positions,
                             const int* item_len, const int* item_tok_off, const int* item_slot, int num_items, int heads,
                             int qk_heads, int key_dim, int value_dim, int taps, float q_scale, float unit_eps, float eps,
                             int dtype, hipStream_t stream) {
    const DeltaShape sh{heads, qk_heads, key_dim, value_dim, taps};
    if (delta_check(sh, stride, slot_stride, eps, unit_eps)) return 1;
    ST_CHECK(num_items >= 0 && num_items <= 65535, "delta_step: %d items", num_items);
    if (num_items == 0) return 0;
    ST_CHECK(out && proj && state && taps_w && a_log && dt_bias && gain && positions && item_len && item_tok_off && item_slot,
             "delta_step: null operand");
    const bool vec = value_dim % 4 == 0 && slot_stride % 4 == 0 && ((uintptr_t)state & 15) == 0;
    const int cols = value_dim / (vec ? 4 : 1), pieces = cols * key_dim;
    int threads = 256;
    while (threads < 1024 && threads * (vec ? 4 : 16) < pieces) threads <<= 1;
    const int lanes = threads / cols < key_dim ? threads / cols : key_dim;
    const int np = (key_dim + lanes - 1) / lanes;
    const size_t lds = sizeof(float) * ((size_t)2 * key_dim + 2 * value_dim + 2 * (size_t)lanes * value_dim + 48);
    ST_CHECK(np <= (vec ? 16 : 64) && lds <= 64 * 1024, "delta_step: %d pieces a thread, %zu bytes of LDS", np, lds);
    const dim3 grid(heads, num_items);
#define ST_DS(T, V, NP)                                                                                                \
    delta_step_kernel<T, V, NP><<<grid, threads, lds, stream>>>((T*)out, proj, stride, state, slot_stride, taps_w, a_log, dt_bias, \
        gain, positions, item_len, item_tok_off, item_slot, sh, q_scale, unit_eps, eps, lanes)
#define ST_DS_T(T) do { if (vec) { if (np <= 4) ST_DS(T, 4, 4); else ST_DS(T, 4, 16); }                                 \
                        else { if (np <= 16) ST_DS(T, 1, 16); else ST_DS(T, 1, 64); } } while (0)
    if (dtype == kF32) ST_DS_T(float);
    else if (dtype == kBF16) ST_DS_T(bf16_t);
    else ST_CHECK(false, "delta_step: unknown dtype %d", dtype);
#undef ST_DS_T
#undef ST_DS
    ST_LAUNCH_CHECK("delta_step");
    return 0;
}

// Items of any length.  Scratch: qkv [rows, channels], gates [rows, 2 heads], wv [chunks, heads, 64, dv], wk [chunks, heads,
// 64, dk], kt [chunks, heads, dk, 64], fall [chunks, heads], start [chunks, heads, dk, dv]; chunks >= rows / 64 + items.
extern "C" int st_delta_chunks(void* out, const float* proj, int64_t stride, float* state, int64_t slot_stride, const float* taps_w,
                               const float* a_log, const float* dt_bias, const float* gain, const int* token_item,
                               const int* positions, const int* item_len, const int* item_tok_off, const int* item_slot,
                               int num_items, int num_rows, int heads, int qk_heads, int key_dim, int value_dim, int taps,
                               float q_scale, float unit_eps, float eps, float* qkv, float* gates, float* wv, float* wk, float* kt,
                               float* fall, float* start, int64_t scratch_chunks, int dtype, hipStream_t stream) {
    const DeltaShape sh{heads, qk_heads, key_dim, value_dim, taps};
    if (delta_check(sh, stride, slot_stride, eps, unit_eps)) return 1;
    ST_CHECK(num_items >= 0 && num_rows >= 0, "delta_chunks: bad sizes");
    if (num_items == 0 || num_rows == 0) return 0;
    ST_CHECK(out && proj && state && taps_w && a_log && dt_bias && gain && token_item && positions && item_len && item_tok_off &&
             item_slot && qkv && gates && wv && wk && kt && fall && start, "delta_chunks: null operand");
    ST_CHECK(dtype == kF32 || dtype == kBF16, "delta_chunks: unknown dtype %d", dtype);
    const int64_t chunks = num_rows / kChunkRows + num_items;  // every item's last chunk may be a short one
    ST_CHECK(scratch_chunks >= chunks, "delta_chunks: scratch for %lld chunks, %lld needed", (long long)scratch_chunks, (long long)chunks);
    ST_CHECK(chunks <= 65535 && num_items <= 65535, "delta_chunks: too many chunks or items");
    const int seg = key_dim <= 64 ? 1 : key_dim <= 128 ? 2 : 4;
    const int units = delta_head_units(sh, seg) + (heads * value_dim + 255) / 256 + 1;
    const dim3 grid_in((num_rows + kInputRows - 1) / kInputRows, (units + 3) / 4);
#define ST_DI(TM, SEG)                                                                                                 \
    delta_inputs_kernel<TM, SEG><<<grid_in, 256, 0, stream>>>(qkv, gates, proj, stride, state, slot_stride, taps_w, a_log, dt_bias, \
        token_item, positions, item_tok_off, item_slot, num_rows, units, sh, q_scale, unit_eps)
#define ST_DI_S(TM) do { if (seg == 1) ST_DI(TM, 1); else if (seg == 2) ST_DI(TM, 2); else ST_DI(TM, 4); } while (0)
    if (taps <= 4) ST_DI_S(4); else ST_DI_S(8);
#undef ST_DI_S
#undef ST_DI
    ST_LAUNCH_CHECK("delta_chunks (inputs)");
    // 16-byte loads where every section of a row and every row of the scratch starts on a 16-byte border
    const bool vec = key_dim % 4 == 0 && value_dim % 4 == 0 && stride % 4 == 0 &&
                     (((uintptr_t)proj | (uintptr_t)qkv | (uintptr_t)wv | (uintptr_t)start | (uintptr_t)gain) & 15) == 0;
    ST_CHECK((((uintptr_t)wk | (uintptr_t)kt) & 15) == 0, "delta_chunks: scratch is 16-byte aligned");
    const dim3 grid(heads, (unsigned)chunks);
#define ST_DP2(KQ, VEC)                                                                                                \
    do {                                                                                                               \
        auto kernel = delta_prep_kernel<KQ, VEC>;                                                                       \
        constexpr size_t lds = sizeof(double) * kChunkRows + sizeof(float) * (size_t)(kChunkRows + kChunkRows * (4 * KQ + 4) + kChunkRows * (kChunkRows + 4)); \
        if (delta_raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;                                      \
        kernel<<<grid, 256, lds, stream>>>(wv, wk, kt, fall, qkv, gates, item_len, item_tok_off, item_slot, num_items, sh); \
    } while (0)
#define ST_DP(KQ) do { if (vec) ST_DP2(KQ, true); else ST_DP2(KQ, false); } while (0)
    if (key_dim <= 16) ST_DP(4);
    else if (key_dim <= 32) ST_DP(8);
    else if (key_dim <= 64) ST_DP(16);
    else if (key_dim <= 128) ST_DP(32);
    else ST_DP(64);
#undef ST_DP
#undef ST_DP2
    ST_LAUNCH_CHECK("delta_chunks (prep)");
    const dim3 grid_c(heads, (value_dim + 15) / 16, num_items);
#define ST_DC(KT, AHEAD) delta_carry_kernel<KT, AHEAD><<<grid_c, 256, 0, stream>>>(wv, wk, kt, fall, start, state, slot_stride, item_len, item_slot, sh)
    if (key_dim <= 16) ST_DC(1, 4);
    else if (key_dim <= 32) ST_DC(2, 4);
    else if (key_dim <= 64) ST_DC(4, 4);
    else if (key_dim <= 128) ST_DC(8, 2);
    else ST_DC(16, 1);
#undef ST_DC
    ST_LAUNCH_CHECK("delta_chunks (carry)");
#define ST_DO_E(T, KQ, NV, VEC)                                                                                        \
    do {                                                                                                               \
        auto kernel = delta_out_kernel<T, KQ, NV, VEC>;                                                                 \
        constexpr size_t lds = DeltaOutLds<KQ, NV>::bytes;                                                              \
        if (delta_raise_lds(reinterpret_cast<const void*>(kernel), lds)) return 1;                                      \
        kernel<<<grid, 256, lds, stream>>>((T*)out, proj, stride, qkv, gates, wv, start, state, slot_stride, gain, positions, \
            item_len, item_tok_off, item_slot, num_items, sh, eps);                                                    \
    } while (0)
#define ST_DO(T, KQ, NV) do { if (vec) ST_DO_E(T, KQ, NV, true); else ST_DO_E(T, KQ, NV, false); } while (0)
#define ST_DO_V(T, KQ) do { if (value_dim <= 64) ST_DO(T, KQ, 4); else if (value_dim <= 128) ST_DO(T, KQ, 8); else ST_DO(T, KQ, 16); } while (0)
#define ST_DO_K(T) do { if (key_dim <= 32) ST_DO_V(T, 8); else if (key_dim <= 64) ST_DO_V(T, 16); else if (key_dim <= 128) ST_DO_V(T, 32); else ST_DO_V(T, 64); } while (0)
    if (dtype == kF32) ST_DO_K(float); else ST_DO_K(bf16_t);
#undef ST_DO_K
#undef ST_DO_V
#undef ST_DO
#undef ST_DO_E
    ST_LAUNCH_CHECK("delta_chunks (outputs)");
    return 0;
}
