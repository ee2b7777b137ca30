// Linear attention with decays: a memory S [key channel i, value channel j] per request and head,
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T        o_t = S_t^T q_t
// where the decay a_t is one number a key channel that depends on the token,
//   a = sigmoid(z)^(1/tau),   z = W_out (W_in x) + bias   (W_in x arrives as `low`),
// or one fixed number a head.  q, k and v are columns of a packed row of the projections, taken as
// they are or through silu; q is multiplied by q_scale.  Everything here is float32; the element
// type T only says how the projections' results are read and the mixer's outputs written.
//
// A step is a flat batch of requests: request s brings the tokens cu[s] .. cu[s + 1] - 1 and keeps
// its memory in row seq_slots[s] of S [slots, heads, d, dv].
//
// Portions are walked in chunks of 16 tokens.  With b_t the sum of ln a over the chunk's tokens up
// to t (per key channel), and t' <= t two of its tokens,
//   o_t = S_0^T (q_t e^(b_t)) + sum_t' A_tt' v_t'        A_tt' = sum_i q_ti k_t'i e^(b_ti - b_t'i)
//   S_1 = diag(e^(b_last)) S_0 + sum_t (k_t e^(b_last - b_t)) v_t^T.
// No exponent is positive, so nothing overflows whatever the decays are.  A first kernel, a
// workgroup a (chunk, head), forms the three sets of factors; the second walks a request's chunks
// with the memory in the registers of the matrix instruction (v_mfma_f32_16x16x4_f32: true
// 32-bit) and never moves it: a lane holds rows 4g .. 4g + 3 of a block of 16 rows in one column,
// which is the result's layout of the update and, with the sum over the rows taken in that order,
// the operand's layout of the read-out.
//
// A step of single tokens streams every memory through once and finishes the heads in place.
#include "common.h"

namespace linattn {

constexpr int CT = 16;            // tokens of a chunk
constexpr int MAX_D = 256;        // key channels of a head
constexpr int MAX_DV = 512;       // value channels of a head
constexpr int XCDS = 8;
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <typename T>
struct alignas(sizeof(T) * 4) Quad {
    T v[4];
};

// exponentials: the library's in a float32 engine, the hardware's (of base 2, in float32) in a
// bfloat16 one
template <typename T>
__device__ inline float fexp(float x);
template <>
__device__ inline float fexp<float>(float x) {
    return expf(x);
}
template <>
__device__ inline float fexp<bf16_t>(float x) {
    return __builtin_amdgcn_exp2f(1.4426950408889634f * x);
}

__device__ inline float silu(float z) { return z / (1.f + expf(-z)); }
__device__ inline float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// what the kernels read of a token
template <typename T>
struct Rows {
    const T* packed;
    int width, q_col, k_col, v_col;
    int silu;       // q, k and v pass silu
    float q_scale;
};
template <typename T>
__device__ inline float input(const Rows<T>& in, int t, int col) {
    const float x = to_float(in.packed[(size_t)t * in.width + col]);
    return in.silu ? linattn::silu(x) : x;
}

// where a token's decays come from
struct Decays {
    const float* low;    // [tokens, low_stride], the first `rank` columns: W_in x
    const float* out_t;  // [rank, heads * d]: W_out transposed; null: fixed decays
    const float* bias;   // [heads * d]
    const float* fixed;  // [heads]: ln a
    int low_stride, rank;
    float inv_tau;
};

// --------------------------------------------------------------------------- //
// The factors of a chunk: Q [16][DP] = q e^(b_t), KT [DP][16] = k e^(b_last - b_t), G [DP] =
// e^(b_last), A [16][16] (0 above the diagonal), where DP is d rounded up to whole blocks of 16
// rows and what lies beyond d or the chunk's tokens is zero.
// chunks: [n][4] = request, first token, tokens, unused.
// --------------------------------------------------------------------------- //
template <typename T, bool CHANNEL>
__global__ __launch_bounds__(256) void chunk_factors_kernel(Rows<T> in, Decays dec, const int* __restrict__ chunks,
                                                            float* __restrict__ Q, float* __restrict__ KT,
                                                            float* __restrict__ G, float* __restrict__ A, int heads,
                                                            int d, int DP) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int chunk = blockIdx.x, h = blockIdx.y;
    const int t0 = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2];
    const int P = DP + 4;  // pitch of a token's channels
    float* sq = lds;
    float* sk = sq + CT * P;
    float* sb = sk + CT * P;                       // CHANNEL: the sums of ln a
    float* red = CHANNEL ? sb + CT * P : sb;       // [4][16][16]
    float* slow = red + 4 * CT * CT;               // CHANNEL: [16][rank]
    const int tid = threadIdx.x, lane = tid & (RL_WAVE - 1), wave = tid / RL_WAVE;
    for (int idx = tid; idx < CT * DP; idx += 256) {
        const int t = idx / DP, i = idx - t * DP;
        const bool ok = t < n && i < d;
        sq[t * P + i] = ok ? input(in, t0 + t, in.q_col + h * d + i) * in.q_scale : 0.f;
        sk[t * P + i] = ok ? input(in, t0 + t, in.k_col + h * d + i) : 0.f;
    }
    const float fixed = CHANNEL ? 0.f : dec.fixed[h];
    if constexpr (CHANNEL) {
        for (int idx = tid; idx < CT * dec.rank; idx += 256) {
            const int t = idx / dec.rank, r = idx - t * dec.rank;
            slow[idx] = t < n ? dec.low[(size_t)(t0 + t) * dec.low_stride + r] : 0.f;
        }
        __syncthreads();
        // a thread takes a channel of eight tokens, so that an entry of W_out serves eight sums
        for (int item = tid; item < 2 * DP; item += 256) {
            const int half = item / DP, i = item - half * DP;
            if (i >= d) {
                for (int t = 0; t < CT / 2; ++t) sb[(half * (CT / 2) + t) * P + i] = 0.f;
                continue;
            }
            float z[CT / 2];
            const float b = dec.bias[h * d + i];
#pragma unroll
            for (int t = 0; t < CT / 2; ++t) z[t] = 0.f;
            const float* col = dec.out_t + h * d + i;
            const float* lrow = slow + half * (CT / 2) * dec.rank;
#pragma unroll 4
            for (int r = 0; r < dec.rank; ++r) {
                const float w = col[(size_t)r * heads * d];
#pragma unroll
                for (int t = 0; t < CT / 2; ++t) z[t] = fmaf(w, lrow[t * dec.rank + r], z[t]);
            }
#pragma unroll
            for (int t = 0; t < CT / 2; ++t) {
                const int tt = half * (CT / 2) + t;
                sb[tt * P + i] = tt < n ? log_sigmoid(z[t] + b) * dec.inv_tau : 0.f;
            }
        }
        __syncthreads();
        for (int i = tid; i < DP; i += 256) {
            float sum = 0.f;
#pragma unroll
            for (int t = 0; t < CT; ++t) {
                sum += sb[t * P + i];
                sb[t * P + i] = sum;
            }
        }
    }
    __syncthreads();
    const size_t cb = (size_t)chunk * heads + h;
    for (int idx = tid; idx < CT * DP; idx += 256) {
        const int t = idx / DP, i = idx - t * DP;
        const float b = CHANNEL ? sb[t * P + i] : fixed * (float)(t + 1);
        Q[cb * CT * DP + idx] = sq[t * P + i] * fexp<T>(b);
    }
    for (int idx = tid; idx < CT * DP; idx += 256) {
        const int i = idx / CT, t = idx & (CT - 1);
        // (t beyond the chunk's tokens: its key is zero, and the exponent is kept from growing)
        const float b = CHANNEL ? sb[(CT - 1) * P + i] - sb[t * P + i] : fixed * (float)max(n - 1 - t, 0);
        KT[cb * CT * DP + idx] = sk[t * P + i] * fexp<T>(b);
    }
    for (int i = tid; i < DP; i += 256) G[cb * DP + i] = fexp<T>(CHANNEL ? sb[(CT - 1) * P + i] : fixed * (float)n);
    // A: a lane takes two by two tokens, a wave a quarter of the channels
    const int ta = 2 * (lane >> 3), sa = 2 * (lane & 7);
    float acc[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
    if (sa <= ta) {
        for (int i = wave * (DP / 4); i < (wave + 1) * (DP / 4); i += 4) {
            f32x4 q[2], k[2], bt[2], bs[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                q[e] = *reinterpret_cast<const f32x4*>(sq + (ta + e) * P + i);
                k[e] = *reinterpret_cast<const f32x4*>(sk + (sa + e) * P + i);
                if constexpr (CHANNEL) {
                    bt[e] = *reinterpret_cast<const f32x4*>(sb + (ta + e) * P + i);
                    bs[e] = *reinterpret_cast<const f32x4*>(sb + (sa + e) * P + i);
                }
            }
#pragma unroll
            for (int a = 0; a < 2; ++a)
#pragma unroll
                for (int s = 0; s < 2; ++s)
#pragma unroll
                    for (int c = 0; c < 4; ++c) {
                        float x = q[a][c] * k[s][c];
                        // (a pair above the diagonal is not used; its exponent would be positive)
                        if constexpr (CHANNEL) x *= fexp<T>(fminf(bt[a][c] - bs[s][c], 0.f));
                        acc[a][s] += x;
                    }
        }
    }
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int s = 0; s < 2; ++s) red[(wave * CT + ta + a) * CT + sa + s] = acc[a][s];
    __syncthreads();
    const int t = tid / CT, s = tid % CT;
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum += red[(w * CT + t) * CT + s];
    if constexpr (!CHANNEL) sum *= fexp<T>(fixed * (float)max(t - s, 0));
    A[cb * CT * CT + tid] = s <= t ? sum : 0.f;
}

// --------------------------------------------------------------------------- //
// The walk over a request's chunks.  A workgroup of four waves takes 16 columns of a head; the
// blocks of 16 rows are dealt to the waves, RB at most each, so that a wave's own chain of matrix
// instructions is short.  The read-outs' shares of the waves are added through LDS behind the
// update, which does not wait for them.  Operands of the next two chunks travel meanwhile.
// seq_chunks: [requests][2] = first chunk, chunks.
// --------------------------------------------------------------------------- //
template <typename T, int RB>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void chunk_walk_kernel(
    Rows<T> in, const float* __restrict__ Q, const float* __restrict__ KT, const float* __restrict__ G,
    const float* __restrict__ A, const int* __restrict__ cu, const int* __restrict__ seq_slots,
    const int* __restrict__ seq_chunks, float* __restrict__ S, float* __restrict__ raw, int num_seqs, int heads, int d,
    int DP, int dv, int col_groups) {
    // the column groups of a (request, head) read the same factors: they go to one XCD, whose L2 holds them
    const int per_xcd = gridDim.x / XCDS;  // (the launch is a multiple)
    const int work = (blockIdx.x % XCDS) * per_xcd + blockIdx.x / XCDS;
    if (work >= num_seqs * heads * col_groups) return;  // whole workgroups leave
    const int pair = work / col_groups;
    const int s = pair / heads, h = pair - s * heads;
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = threadIdx.x / RL_WAVE;
    const int r16 = lane & 15, g = lane >> 4;
    const int j0 = (work - pair * col_groups) * 16;
    const int j = min(j0 + r16, dv - 1);
    const int t0 = cu[s], t1 = cu[s + 1];
    const int c0 = seq_chunks[2 * s], nc = seq_chunks[2 * s + 1];
    const int NB = DP / 16;
    __shared__ float red[2][4][CT][CT + 1];

    f32x4 st[RB];
    float* Sp = S + ((size_t)seq_slots[s] * heads + h) * d * dv;
#pragma unroll
    for (int m = 0; m < RB; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = 16 * (wave + 4 * m) + 4 * g + r;
            st[m][r] = i < d ? Sp[(size_t)i * dv + j] : 0.f;
        }

    struct Operands {
        f32x4 q[RB], k[RB], decay[RB];
        float a;
        T v[4];
    };
    auto load = [&](int c, Operands& x) {
        const size_t cb = (size_t)(c0 + c) * heads + h;
#pragma unroll
        for (int m = 0; m < RB; ++m) {
            const int rb = min(wave + 4 * m, NB - 1);
            x.q[m] = *reinterpret_cast<const f32x4*>(Q + (cb * CT + r16) * DP + 16 * rb + 4 * g);
            x.k[m] = *reinterpret_cast<const f32x4*>(KT + (cb * DP + 16 * rb + r16) * CT + 4 * g);
            x.decay[m] = *reinterpret_cast<const f32x4*>(G + cb * DP + 16 * rb + 4 * g);
        }
        x.a = A[cb * CT * CT + r16 * CT + 4 * g + wave];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            // (beyond the portion a real row, which meets zeros)
            const int t = min(t0 + c * CT + 4 * g + r, t1 - 1);
            x.v[r] = in.packed[(size_t)t * in.width + in.v_col + h * dv + j];
        }
    };
    auto walk = [&](int c, const Operands& x) {
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            v[r] = to_float(x.v[r]);
            if (in.silu) v[r] = linattn::silu(v[r]);
        }
        // the chunk's own pairs: wave w takes tokens 4g + w
        const float mine = wave == 0 ? v[0] : (wave == 1 ? v[1] : (wave == 2 ? v[2] : v[3]));
        f32x4 o = (f32x4){0.f, 0.f, 0.f, 0.f};
        f32x4 o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a, mine, o, 0, 0, 0);
#pragma unroll
        for (int m = 0; m < RB; ++m) {
            if (wave + 4 * m < NB) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if (r & 1)
                        o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m][r], st[m][r], o2, 0, 0, 0);
                    else
                        o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m][r], st[m][r], o, 0, 0, 0);
                }
            }
        }
#pragma unroll
        for (int m = 0; m < RB; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) st[m][r] *= x.decay[m][r];
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int m = 0; m < RB; ++m)
                if (wave + 4 * m < NB) st[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[m][r], v[r], st[m], 0, 0, 0);
        float(*buf)[CT][CT + 1] = red[c & 1];
#pragma unroll
        for (int r = 0; r < 4; ++r) buf[wave][4 * g + r][r16] = o[r] + o2[r];
        // one barrier a chunk: the other buffer is written next, and this one again only after
        // every wave has passed the next barrier
        __syncthreads();
        const int tt = threadIdx.x / 16, jj = threadIdx.x % 16;
        const int t = t0 + c * CT + tt;
        if (t < t1 && j0 + jj < dv)
            raw[(size_t)t * heads * dv + h * dv + j0 + jj] =
                (buf[0][tt][jj] + buf[1][tt][jj]) + (buf[2][tt][jj] + buf[3][tt][jj]);
    };
    Operands x[3];
    load(0, x[0]);
    load(min(1, nc - 1), x[1]);
    for (int c = 0; c < nc; c += 3) {
#pragma unroll
        for (int u = 0; u < 3; ++u) {
            if (c + u < nc) {
                load(min(c + u + 2, nc - 1), x[(u + 2) % 3]);
                __builtin_amdgcn_sched_barrier(0);
                walk(c + u, x[u]);
            }
        }
    }
#pragma unroll
    for (int m = 0; m < RB; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = 16 * (wave + 4 * m) + 4 * g + r;
            if (i < d && j0 + r16 < dv) Sp[(size_t)i * dv + j0 + r16] = st[m][r];
        }
}

// --------------------------------------------------------------------------- //
// How an output leaves: o (float32) in parts (every head, or the whole row), each divided by its
// root mean square, times a weight and the gate (silu or sigmoid of a column of the packed row).
// --------------------------------------------------------------------------- //
template <typename T>
struct Finish {
    const float* weight;  // [inner], or [part] for every part
    const T* gate;        // first column of the gate in rows of gate_width
    T* out;               // first column of the output in rows of out_width
    int gate_width, out_width;
    int shared_w;
    int sigmoid_gate;
    float eps;
};
template <typename T>
__device__ inline float gate_of(const Finish<T>& f, int t, int col) {
    const float z = to_float(f.gate[(size_t)t * f.gate_width + col]);
    return f.sigmoid_gate ? 1.f / (1.f + expf(-z)) : silu(z);
}

// parts of up to 1024 channels: LPP lanes of a wave a part, four channels a lane at a time
template <typename T, int LPP, bool WHOLE>
__global__ __launch_bounds__(256) void gated_norm_kernel(const float* __restrict__ raw, Finish<T> f, int rows, int parts,
                                                         int size) {
    const int row = (blockIdx.x * 256 + threadIdx.x) / LPP;  // (token, part)
    const int lane = threadIdx.x % LPP;
    const bool live = row < rows;
    const int t = (live ? row : 0) / parts, part = (live ? row : 0) % parts;
    const float* src = raw + ((size_t)t * parts + part) * size;
    float ss = 0.f;
    if constexpr (WHOLE) {
        for (int i = 4 * lane; i < size; i += 4 * LPP) {
            const float4 v = *reinterpret_cast<const float4*>(src + i);
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    } else {
        for (int i = lane; i < size; i += LPP) ss += src[i] * src[i];
    }
#pragma unroll
    for (int o = LPP / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, RL_WAVE);
    if (!live) return;
    const float rr = rsqrtf(ss / (float)size + f.eps);
    const float* w = f.weight + (f.shared_w ? 0 : part * size);
    if constexpr (WHOLE) {
        for (int i = 4 * lane; i < size; i += 4 * LPP) {
            const float4 v = *reinterpret_cast<const float4*>(src + i);
            const float4 wt = *reinterpret_cast<const float4*>(w + i);
            const Quad<T> gq = *reinterpret_cast<const Quad<T>*>(f.gate + (size_t)t * f.gate_width + part * size + i);
            const float x[4] = {v.x * wt.x, v.y * wt.y, v.z * wt.z, v.w * wt.w};
            Quad<T> y;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float z = to_float(gq.v[e]);
                y.v[e] = from_float<T>(x[e] * rr * (f.sigmoid_gate ? 1.f / (1.f + expf(-z)) : silu(z)));
            }
            *reinterpret_cast<Quad<T>*>(f.out + (size_t)t * f.out_width + part * size + i) = y;
        }
    } else {
        for (int i = lane; i < size; i += LPP)
            f.out[(size_t)t * f.out_width + part * size + i] =
                from_float<T>(src[i] * w[i] * rr * gate_of(f, t, part * size + i));
    }
}

// wider parts, and rows of a step that has few: a workgroup a part
template <typename T, bool WHOLE>
__global__ __launch_bounds__(512) void gated_norm_row_kernel(const float* __restrict__ raw, Finish<T> f, int parts, int size) {
    __shared__ float scratch[16];
    const int t = blockIdx.x, part = blockIdx.y;
    const float* src = raw + ((size_t)t * parts + part) * size;
    const float* w = f.weight + (f.shared_w ? 0 : part * size);
    float ss = 0.f;
    if constexpr (WHOLE) {
        for (int i = 4 * threadIdx.x; i < size; i += 4 * blockDim.x) {
            const float4 v = *reinterpret_cast<const float4*>(src + i);
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    } else {
        for (int i = threadIdx.x; i < size; i += blockDim.x) ss += src[i] * src[i];
    }
    const float rr = rsqrtf(block_sum(ss, scratch) / (float)size + f.eps);
    if constexpr (WHOLE) {
        for (int i = 4 * threadIdx.x; i < size; i += 4 * blockDim.x) {
            const float4 v = *reinterpret_cast<const float4*>(src + i);
            const float4 wt = *reinterpret_cast<const float4*>(w + i);
            const Quad<T> gq = *reinterpret_cast<const Quad<T>*>(f.gate + (size_t)t * f.gate_width + part * size + i);
            const float x[4] = {v.x * wt.x, v.y * wt.y, v.z * wt.z, v.w * wt.w};
            Quad<T> y;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float z = to_float(gq.v[e]);
                y.v[e] = from_float<T>(x[e] * rr * (f.sigmoid_gate ? 1.f / (1.f + expf(-z)) : silu(z)));
            }
            *reinterpret_cast<Quad<T>*>(f.out + (size_t)t * f.out_width + part * size + i) = y;
        }
    } else {
        for (int i = threadIdx.x; i < size; i += blockDim.x)
            f.out[(size_t)t * f.out_width + part * size + i] =
                from_float<T>(src[i] * w[i] * rr * gate_of(f, t, part * size + i));
    }
}

// --------------------------------------------------------------------------- //
// Single tokens: a workgroup takes a (request, head), its memory goes through once.  Threads lie as
// [row][VEC columns]; a thread's rows of one batch are all asked for before the first is used.  With
// `finish` the head is normed, gated and written here, otherwise o goes to `raw`.
// --------------------------------------------------------------------------- //
constexpr int STEP_THREADS = 512;
constexpr int STEP_BATCH = 8;

template <typename T, bool CHANNEL, int VEC>
__global__ __launch_bounds__(STEP_THREADS) void memory_step_kernel(Rows<T> in, Decays dec,
                                                                   const int* __restrict__ seq_slots,
                                                                   float* __restrict__ S, float* __restrict__ raw,
                                                                   Finish<T> f, int finish, int heads, int d, int dv,
                                                                   int unit_shift) {
    struct alignas(4 * VEC) Pack {
        float v[VEC];
    };
    __shared__ float sq[MAX_D], sk[MAX_D], sa[MAX_D];
    __shared__ Pack red[STEP_THREADS];
    __shared__ float scratch[16];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int units = dv / VEC, lanes = 1 << unit_shift;  // lanes >= units, a power of two
    const int u = tid & (lanes - 1), row = tid >> unit_shift, per_pass = STEP_THREADS >> unit_shift;
    const bool live = u < units;
    float* Sp = S + ((size_t)seq_slots[t] * heads + h) * d * dv + VEC * u;
    // the first batch of rows travels while the token's operands are formed
    Pack s[STEP_BATCH];
    auto fetch = [&](int base) {
#pragma unroll
        for (int b = 0; b < STEP_BATCH; ++b) {
            const int i = base + b * per_pass;
            if (live && i < d) s[b] = *reinterpret_cast<const Pack*>(Sp + (size_t)i * dv);
        }
    };
    fetch(row);
    for (int i = tid; i < d; i += STEP_THREADS) {
        sq[i] = input(in, t, in.q_col + h * d + i) * in.q_scale;
        sk[i] = input(in, t, in.k_col + h * d + i);
        if constexpr (CHANNEL) {
            float z = 0.f;
            const float* low = dec.low + (size_t)t * dec.low_stride;
#pragma unroll 8
            for (int r = 0; r < dec.rank; ++r) z = fmaf(dec.out_t[(size_t)r * heads * d + h * d + i], low[r], z);
            sa[i] = fexp<T>(log_sigmoid(z + dec.bias[h * d + i]) * dec.inv_tau);
        } else {
            sa[i] = fexp<T>(dec.fixed[h]);
        }
    }
    float v[VEC], acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
        v[e] = live ? input(in, t, in.v_col + h * dv + VEC * u + e) : 0.f;
        acc[e] = 0.f;
    }
    __syncthreads();
    for (int base = row; base < d; base += STEP_BATCH * per_pass) {
        if (base != row) fetch(base);
#pragma unroll
        for (int b = 0; b < STEP_BATCH; ++b) {
            const int i = base + b * per_pass;
            if (live && i < d) {
                const float a = sa[i], k = sk[i], q = sq[i];
                Pack next;
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    next.v[e] = fmaf(k, v[e], a * s[b].v[e]);
                    acc[e] = fmaf(q, next.v[e], acc[e]);
                }
                *reinterpret_cast<Pack*>(Sp + (size_t)i * dv) = next;
            }
        }
    }
    Pack mine;
#pragma unroll
    for (int e = 0; e < VEC; ++e) mine.v[e] = acc[e];
    red[tid] = mine;
    __syncthreads();
    // thread j adds column j's shares of the rows
    float o = 0.f;
    if (tid < dv)
        for (int r = 0; r < per_pass; ++r) o += red[(r << unit_shift) + tid / VEC].v[tid % VEC];
    if (!finish) {
        if (tid < dv) raw[((size_t)t * heads + h) * dv + tid] = o;
        return;
    }
    const float rr = rsqrtf(block_sum(o * o, scratch) / (float)dv + f.eps);
    if (tid < dv) {
        const int col = h * dv + tid;
        f.out[(size_t)t * f.out_width + col] =
            from_float<T>(o * f.weight[f.shared_w ? tid : col] * rr * gate_of(f, t, col));
    }
}

template <typename T>
static int launch_gated_norm(const float* raw, const Finish<T>& f, int tokens, int parts, int size, hipStream_t stream) {
    const bool whole = size % 4 == 0 && f.gate_width % 4 == 0 && f.out_width % 4 == 0 &&
                       (uintptr_t)f.gate % (4 * sizeof(T)) == 0 && (uintptr_t)f.out % (4 * sizeof(T)) == 0;
    if (size > 512) {
        dim3 grid(tokens, parts);
        const int threads = size >= 2048 ? 512 : 256;
        if (whole)
            hipLaunchKernelGGL((gated_norm_row_kernel<T, true>), grid, dim3(threads), 0, stream, raw, f, parts, size);
        else
            hipLaunchKernelGGL((gated_norm_row_kernel<T, false>), grid, dim3(threads), 0, stream, raw, f, parts, size);
        return rl_launch_status();
    }
    const int rows = tokens * parts;
#define RL_GATED(LPP)                                                                                                \
    do {                                                                                                             \
        dim3 grid((unsigned)(((long)rows * LPP + 255) / 256));                                                       \
        if (whole)                                                                                                   \
            hipLaunchKernelGGL((gated_norm_kernel<T, LPP, true>), grid, dim3(256), 0, stream, raw, f, rows, parts, size); \
        else                                                                                                         \
            hipLaunchKernelGGL((gated_norm_kernel<T, LPP, false>), grid, dim3(256), 0, stream, raw, f, rows, parts, size); \
    } while (0)
    if (size <= 64)
        RL_GATED(16);
    else if (size <= 128)
        RL_GATED(32);
    else
        RL_GATED(64);
#undef RL_GATED
    return rl_launch_status();
}

template <typename T>
static int launch_scan(const Rows<T>& in, const Decays& dec, const int* chunks, int nchunks, const int* cu,
                       const int* seq_slots, const int* seq_chunks, float* Q, float* KT, float* G, float* A, float* S,
                       float* raw, int num_seqs, int heads, int d, int dv, hipStream_t stream) {
    const int DP = (d + 15) / 16 * 16;
    const bool channel = dec.out_t != nullptr;
    const size_t lds = sizeof(float) * ((size_t)(channel ? 3 : 2) * CT * (DP + 4) + 4 * CT * CT +
                                        (channel ? (size_t)CT * dec.rank : 0));
    if (lds > 156 * 1024) return RL_ERR_ARG;
    auto factors = channel ? chunk_factors_kernel<T, true> : chunk_factors_kernel<T, false>;
    if (lds > 60 * 1024 &&
        hipFuncSetAttribute((const void*)factors, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
        return RL_ERR_LAUNCH;
    hipLaunchKernelGGL(factors, dim3(nchunks, heads), dim3(256), lds, stream, in, dec, chunks, Q, KT, G, A, heads, d, DP);
    const int col_groups = (dv + 15) / 16;
    const long groups = ((long)num_seqs * heads * col_groups + XCDS - 1) / XCDS * XCDS;
    if (groups > 0x7fffffffL) return RL_ERR_ARG;
#define RL_WALK(RB)                                                                                                  \
    hipLaunchKernelGGL((chunk_walk_kernel<T, RB>), dim3((unsigned)groups), dim3(256), 0, stream, in, Q, KT, G, A, cu, \
                       seq_slots, seq_chunks, S, raw, num_seqs, heads, d, DP, dv, col_groups)
    if (DP <= 64)
        RL_WALK(1);
    else if (DP <= 128)
        RL_WALK(2);
    else
        RL_WALK(4);
#undef RL_WALK
    return rl_launch_status();
}

template <typename T>
static int launch_step(const Rows<T>& in, const Decays& dec, const int* seq_slots, float* S, float* raw,
                       const Finish<T>& f, int finish, int tokens, int heads, int d, int dv, hipStream_t stream) {
    const int vec = dv % 4 == 0 ? 4 : 1;
    int shift = 0;
    while ((1 << shift) < dv / vec) ++shift;
    dim3 grid(tokens, heads);
#define RL_STEP(CHANNEL, VEC)                                                                                        \
    hipLaunchKernelGGL((memory_step_kernel<T, CHANNEL, VEC>), grid, dim3(STEP_THREADS), 0, stream, in, dec, seq_slots, \
                       S, raw, f, finish, heads, d, dv, shift)
    if (dec.out_t && vec == 4)
        RL_STEP(true, 4);
    else if (dec.out_t)
        RL_STEP(true, 1);
    else if (vec == 4)
        RL_STEP(false, 4);
    else
        RL_STEP(false, 1);
#undef RL_STEP
    return rl_launch_status();
}

static bool shapes_fit(int width, int q_col, int k_col, int v_col, int heads, int d, int dv, const Decays& dec) {
    if (heads < 1 || heads > 65535 || d < 1 || d > MAX_D || dv < 1 || dv > MAX_DV) return false;
    if (q_col < 0 || k_col < 0 || v_col < 0 || q_col + heads * d > width || k_col + heads * d > width ||
        v_col + heads * dv > width)
        return false;
    if (dec.out_t) return dec.low && dec.bias && dec.rank >= 1 && dec.low_stride >= dec.rank;
    return dec.fixed != nullptr;
}

}  // namespace linattn

extern "C" int rl_linear_attention_max_key_dim() { return linattn::MAX_D; }
extern "C" int rl_linear_attention_max_value_dim() { return linattn::MAX_DV; }
extern "C" int rl_linear_attention_chunk() { return linattn::CT; }

// Portions: raw [tokens, heads * dv] float32 gets o.  Q, KT [chunks, heads, 16 * DP], G [chunks, heads, DP]
// and A [chunks, heads, 256] are scratch.
extern "C" int rl_linear_scan(const void* packed, int width, int q_col, int k_col, int v_col, int silu, float q_scale,
                              const float* low, int low_stride, int rank, const float* out_t, const float* bias,
                              float inv_tau, const float* fixed, const int* chunks, int nchunks, const int* cu,
                              const int* seq_slots, const int* seq_chunks, float* Q, float* KT, float* G, float* A,
                              float* S, float* raw, int num_seqs, int heads, int d, int dv, int act_type,
                              hipStream_t stream) {
    if (nchunks <= 0 || num_seqs <= 0) return RL_OK;
    const linattn::Decays dec = {low, out_t, bias, fixed, low_stride, rank, inv_tau};
    if (!linattn::shapes_fit(width, q_col, k_col, v_col, heads, d, dv, dec)) return RL_ERR_ARG;
    if (act_type == RL_F32) {
        const linattn::Rows<float> in = {(const float*)packed, width, q_col, k_col, v_col, silu, q_scale};
        return linattn::launch_scan<float>(in, dec, chunks, nchunks, cu, seq_slots, seq_chunks, Q, KT, G, A, S, raw,
                                           num_seqs, heads, d, dv, stream);
    }
    if (act_type == RL_BF16) {
        const linattn::Rows<bf16_t> in = {(const bf16_t*)packed, width, q_col, k_col, v_col, silu, q_scale};
        return linattn::launch_scan<bf16_t>(in, dec, chunks, nchunks, cu, seq_slots, seq_chunks, Q, KT, G, A, S, raw,
                                            num_seqs, heads, d, dv, stream);
    }
    return RL_ERR_ARG;
}

// Single tokens, one a request.  With `finish` (parts are heads) `out` gets the finished heads, otherwise raw o.
extern "C" int rl_linear_step(const void* packed, int width, int q_col, int k_col, int v_col, int silu, float q_scale,
                              const float* low, int low_stride, int rank, const float* out_t, const float* bias,
                              float inv_tau, const float* fixed, const int* seq_slots, float* S, float* raw, int finish,
                              const float* norm_w, int shared_w, int gate_col, int sigmoid_gate, float eps, void* out,
                              int out_width, int tokens, int heads, int d, int dv, int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    const linattn::Decays dec = {low, out_t, bias, fixed, low_stride, rank, inv_tau};
    if (!linattn::shapes_fit(width, q_col, k_col, v_col, heads, d, dv, dec)) return RL_ERR_ARG;
    if (finish ? (!norm_w || !out || gate_col < 0 || gate_col + heads * dv > width || out_width < heads * dv) : !raw)
        return RL_ERR_ARG;
    if (act_type == RL_F32) {
        const linattn::Rows<float> in = {(const float*)packed, width, q_col, k_col, v_col, silu, q_scale};
        const linattn::Finish<float> f = {norm_w, (const float*)packed + gate_col, (float*)out, width, out_width,
                                          shared_w, sigmoid_gate, eps};
        return linattn::launch_step<float>(in, dec, seq_slots, S, raw, f, finish, tokens, heads, d, dv, stream);
    }
    if (act_type == RL_BF16) {
        const linattn::Rows<bf16_t> in = {(const bf16_t*)packed, width, q_col, k_col, v_col, silu, q_scale};
        const linattn::Finish<bf16_t> f = {norm_w, (const bf16_t*)packed + gate_col, (bf16_t*)out, width, out_width,
                                           shared_w, sigmoid_gate, eps};
        return linattn::launch_step<bf16_t>(in, dec, seq_slots, S, raw, f, finish, tokens, heads, d, dv, stream);
    }
    return RL_ERR_ARG;
}

// raw [tokens, parts * size] float32; the gate is in the columns from gate_col on of rows of gate_width
extern "C" int rl_gated_norm(const float* raw, const void* gate, int gate_width, int gate_col, const float* norm_w,
                             int shared_w, int sigmoid_gate, float eps, void* out, int out_width, int tokens, int parts,
                             int size, int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (parts < 1 || parts > 65535 || size < 1 || gate_col < 0 || gate_col + parts * size > gate_width ||
        out_width < parts * size || (long)tokens * parts > 0x7fffffffL / 64)
        return RL_ERR_ARG;
    if (act_type == RL_F32) {
        const linattn::Finish<float> f = {norm_w, (const float*)gate + gate_col, (float*)out, gate_width, out_width,
                                          shared_w, sigmoid_gate, eps};
        return linattn::launch_gated_norm<float>(raw, f, tokens, parts, size, stream);
    }
    if (act_type == RL_BF16) {
        const linattn::Finish<bf16_t> f = {norm_w, (const bf16_t*)gate + gate_col, (bf16_t*)out, gate_width, out_width,
                                           shared_w, sigmoid_gate, eps};
        return linattn::launch_gated_norm<bf16_t>(raw, f, tokens, parts, size, stream);
    }
    return RL_ERR_ARG;
}
