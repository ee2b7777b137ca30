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

// (the division likewise)
template <typename T>
__device__ inline float fsigmoid(float z);
template <>
__device__ inline float fsigmoid<float>(float z) {
    return 1.f / (1.f + expf(-z));
}
template <>
__device__ inline float fsigmoid<bf16_t>(float z) {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}
template <typename T>
__device__ inline float silu(float z) {
    return z * fsigmoid<T>(z);
}
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
    return in.silu ? silu<T>(x) : x;
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
// e^(b_last), A [16][16] (0 above the diagonal), where DP is d rounded up to whole blocks of 64
// rows (16 for each of the four waves that walk) and what lies beyond d or the chunk's tokens is zero.
// Q, KT and A lie in the order in which the lanes of the walk hold them as operands, so that a wave
// reads a block of 16 rows as one run of memory: with lane = 16 g + r, Q[block][lane][4] holds channels
// 4g .. 4g + 3 of the block for token r, KT[block][lane][4] tokens 4g .. for channel r, and A[w][lane]
// token r with token 4g + w.
// chunks: [n][4] = request, first token, tokens, unused.
// --------------------------------------------------------------------------- //
template <typename T, bool CHANNEL, int DP>
__global__ __launch_bounds__(256) void chunk_factors_kernel(Rows<T> in, Decays dec, const int* __restrict__ chunks,
                                                            float* __restrict__ Q, float* __restrict__ KT,
                                                            float* __restrict__ G, float* __restrict__ A, int heads,
                                                            int d) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    constexpr int P = DP + 4;  // pitch of a token's channels
    const int chunk = blockIdx.x, h = blockIdx.y;
    const int t0 = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2];
    float* sq = lds;
    float* sk = sq + CT * P;
    float* sb = sk + CT * P;                       // CHANNEL: the sums of ln a, and a itself
    float* sa = sb + CT * P;
    float* red = CHANNEL ? sa + CT * P : sb;       // [4][16][16]
    float* slow = red + 4 * CT * CT;               // CHANNEL: [16][rank up to a multiple of 4]
    const int tid = threadIdx.x, lane = tid & (RL_WAVE - 1), wave = tid / RL_WAVE;
    // every thread's elements are asked for together, without a condition (a real element where there is none)
    constexpr int PER = CT * DP / 256;
    T pq[PER], pk[PER];
#pragma unroll
    for (int e = 0; e < PER; ++e) {
        const int idx = e * 256 + tid, t = min(idx / DP, n - 1), i = min(idx % DP, d - 1);
        const T* row = in.packed + (size_t)(t0 + t) * in.width + h * d + i;
        pq[e] = row[in.q_col];
        pk[e] = row[in.k_col];
    }
    const float fixed = CHANNEL ? 0.f : dec.fixed[h];
    const int pitch = (dec.rank + 3) & ~3;
    if constexpr (CHANNEL) {
        for (int idx = tid; idx < CT * pitch; idx += 256) {
            const int t = idx / pitch, r = idx - t * pitch;
            slow[idx] = t < n && r < dec.rank ? dec.low[(size_t)(t0 + t) * dec.low_stride + r] : 0.f;
        }
    }
#pragma unroll
    for (int e = 0; e < PER; ++e) {
        const int idx = e * 256 + tid, t = idx / DP, i = idx % DP;
        const bool ok = t < n && i < d;
        float q = to_float(pq[e]), k = to_float(pk[e]);
        if (in.silu) {
            q = silu<T>(q);
            k = silu<T>(k);
        }
        sq[t * P + i] = ok ? q * in.q_scale : 0.f;
        sk[t * P + i] = ok ? k : 0.f;
    }
    if constexpr (CHANNEL) {
        __syncthreads();
        // a thread takes a channel of TPT tokens, so that an entry of W_out serves as many sums
        constexpr int PARTS = DP >= 256 ? 1 : 256 / DP, TPT = CT / PARTS;
        for (int item = tid; item < PARTS * DP; item += 256) {
            const int part = item / DP, i = item % DP, ic = min(i, d - 1);
            float z[TPT];
            const float b = dec.bias[h * d + ic];
#pragma unroll
            for (int t = 0; t < TPT; ++t) z[t] = 0.f;
            const float* col = dec.out_t + h * d + ic;
            const float* lrow = slow + part * TPT * pitch;
            for (int r = 0; r < dec.rank; r += 4) {
                float w[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) w[e] = col[(size_t)min(r + e, dec.rank - 1) * heads * d];  // (beyond: times 0)
#pragma unroll
                for (int t = 0; t < TPT; ++t) {
                    const f32x4 l = *reinterpret_cast<const f32x4*>(lrow + t * pitch + r);
                    z[t] = fmaf(w[3], l[3], fmaf(w[2], l[2], fmaf(w[1], l[1], fmaf(w[0], l[0], z[t]))));
                }
            }
#pragma unroll
            for (int t = 0; t < TPT; ++t) {
                const int tt = part * TPT + t;
                const float la = tt < n && i < d ? log_sigmoid(z[t] + b) * dec.inv_tau : 0.f;
                sb[tt * P + i] = la;
                sa[tt * P + i] = fexp<T>(la);
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
    const int r16 = lane & 15, g = lane >> 4;
#pragma unroll
    for (int e = 0; e < PER / 4; ++e) {
        const int block = e * 4 + wave, t = r16, i = 16 * block + 4 * g;
        const f32x4 q = *reinterpret_cast<const f32x4*>(sq + t * P + i);
        f32x4 o;
        if constexpr (CHANNEL) {
            const f32x4 b = *reinterpret_cast<const f32x4*>(sb + t * P + i);
#pragma unroll
            for (int c = 0; c < 4; ++c) o[c] = q[c] * fexp<T>(b[c]);
        } else {
            o = q * fexp<T>(fixed * (float)(t + 1));
        }
        *reinterpret_cast<f32x4*>(Q + cb * CT * DP + 4 * (block * RL_WAVE + lane)) = o;
    }
#pragma unroll
    for (int e = 0; e < PER / 4; ++e) {
        const int block = e * 4 + wave, t = 4 * g, i = 16 * block + r16;
        const float last = CHANNEL ? sb[(CT - 1) * P + i] : 0.f;
        f32x4 o;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            // (t beyond the chunk's tokens: its key is zero, and the exponent is kept from growing)
            const float b = CHANNEL ? last - sb[(t + c) * P + i] : fixed * (float)max(n - 1 - t - c, 0);
            o[c] = sk[(t + c) * P + i] * fexp<T>(b);
        }
        *reinterpret_cast<f32x4*>(KT + cb * CT * DP + 4 * (block * RL_WAVE + lane)) = o;
    }
    for (int i = tid; i < DP; i += 256) G[cb * DP + i] = fexp<T>(CHANNEL ? sb[(CT - 1) * P + i] : fixed * (float)n);
    // A: a lane takes two by two tokens (t, t + 1 with s, s + 1), a wave a quarter of the channels.  One
    // exponential serves the four pairs: with E = e^(b_t - b_(s+1)), the others are E a_(s+1), E a_(t+1)
    // and E a_(s+1) a_(t+1); on the diagonal they are 1 and a_(t+1).
    const int ta = 2 * (lane >> 3), s0 = 2 * (lane & 7);
    const bool diagonal = s0 == ta;
    float acc[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
    if (s0 <= ta) {
#pragma unroll 2
        for (int i = wave * (DP / 4); i < (wave + 1) * (DP / 4); i += 4) {
            f32x4 q[2], k[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                q[e] = *reinterpret_cast<const f32x4*>(sq + (ta + e) * P + i);
                k[e] = *reinterpret_cast<const f32x4*>(sk + (s0 + e) * P + i);
            }
            if constexpr (CHANNEL) {
                const f32x4 bt = *reinterpret_cast<const f32x4*>(sb + ta * P + i);
                const f32x4 bs = *reinterpret_cast<const f32x4*>(sb + (s0 + 1) * P + i);
                const f32x4 at = *reinterpret_cast<const f32x4*>(sa + (ta + 1) * P + i);
                const f32x4 as = *reinterpret_cast<const f32x4*>(sa + (s0 + 1) * P + i);
#pragma unroll
                for (int c = 0; c < 4; ++c) {
                    const float e01 = fexp<T>(fminf(bt[c] - bs[c], 0.f));
                    const float e00 = diagonal ? 1.f : e01 * as[c];
                    const float e11 = diagonal ? 1.f : e01 * at[c];
                    acc[0][0] = fmaf(q[0][c] * k[0][c], e00, acc[0][0]);
                    acc[0][1] = fmaf(q[0][c] * k[1][c], e01, acc[0][1]);  // (not used on the diagonal)
                    acc[1][0] = fmaf(q[1][c] * k[0][c], e00 * at[c], acc[1][0]);
                    acc[1][1] = fmaf(q[1][c] * k[1][c], e11, acc[1][1]);
                }
            } else {
#pragma unroll
                for (int c = 0; c < 4; ++c)
#pragma unroll
                    for (int a = 0; a < 2; ++a)
#pragma unroll
                        for (int s = 0; s < 2; ++s) acc[a][s] = fmaf(q[a][c], k[s][c], acc[a][s]);
            }
        }
    }
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int s = 0; s < 2; ++s) red[(wave * CT + ta + a) * CT + s0 + s] = acc[a][s];
    __syncthreads();
    const int t = r16, s = 4 * g + wave;
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum += red[(w * CT + t) * CT + s];
    if constexpr (!CHANNEL) sum *= fexp<T>(fixed * (float)max(t - s, 0));
    A[cb * CT * CT + tid] = s <= t ? sum : 0.f;
}

// --------------------------------------------------------------------------- //
// The walk over a request's chunks.  A workgroup of four waves takes 16 columns of a head; the
// blocks of 16 rows are dealt to the waves, RB at most each, so that a wave's own chain of matrix
// instructions is short.  The read-outs' shares of the waves meet in LDS and are added and stored while
// the next chunk is multiplied.  Operands of the next chunks travel meanwhile.  A wave is alone on
// its SIMD, so what is not a matrix instruction is to fit between two of them: everything is read
// through buffer resources, whose loads take a constant lane offset and a uniform one, and whose bounds
// stand for the ends of the portion and of the head (reads beyond give zeros, writes are dropped).
// seq_chunks: [requests][2] = first chunk, chunks.
// --------------------------------------------------------------------------- //
constexpr int walk_buffers(int rb) { return rb <= 2 ? 6 : 4; }  // as the registers hold

__device__ inline __amdgpu_buffer_rsrc_t buffer_of(const void* p, size_t bytes) {
    return __builtin_amdgcn_make_buffer_rsrc(const_cast<void*>(p), 0, (int)(unsigned)min(bytes, (size_t)0xfffffffcu), 0x00027000);
}
__device__ inline f32x4 load4(__amdgpu_buffer_rsrc_t r, int lane_bytes, int bytes) {
    return __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(r, lane_bytes, bytes, 0));
}
template <typename T>
__device__ inline T load1(__amdgpu_buffer_rsrc_t r, int lane_bytes, int bytes);
template <>
__device__ inline float load1<float>(__amdgpu_buffer_rsrc_t r, int lane_bytes, int bytes) {
    return __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(r, lane_bytes, bytes, 0));
}
template <>
__device__ inline bf16_t load1<bf16_t>(__amdgpu_buffer_rsrc_t r, int lane_bytes, int bytes) {
    return bf16_t{__builtin_amdgcn_raw_buffer_load_b16(r, lane_bytes, bytes, 0)};
}

template <typename T, int RB, bool SILU>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void chunk_walk_kernel(
    Rows<T> in, const float* __restrict__ Q, const float* __restrict__ KT, const float* __restrict__ G,
    const float* __restrict__ A, const int* __restrict__ cu, const int* __restrict__ seq_slots,
    const int* __restrict__ seq_chunks, float* __restrict__ S, float* __restrict__ raw, int num_seqs, int heads, int d,
    int dv, int col_groups) {
    constexpr int DP = 64 * RB;
    // the column groups of a (request, head) read the same factors: they go to one XCD, whose L2 holds them
    const int per_xcd = gridDim.x / XCDS;  // (the launch is a multiple)
    const int work = (blockIdx.x % XCDS) * per_xcd + blockIdx.x / XCDS;
    if (work >= num_seqs * heads * col_groups) return;  // whole workgroups leave
    const int pair = work / col_groups;
    const int s = pair / heads, h = pair - s * heads;
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / RL_WAVE);
    const int r16 = lane & 15, g = lane >> 4;
    const int j0 = (work - pair * col_groups) * 16;
    const int j = min(j0 + r16, dv - 1);
    const int t0 = cu[s], t1 = cu[s + 1];
    const int c0 = seq_chunks[2 * s], nc = seq_chunks[2 * s + 1];
    __shared__ float red[2][4][CT][CT + 1], sv[2][CT][CT + 1];

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
        T v;  // the value that this thread brings to LDS: token threadIdx.x / 16, column threadIdx.x % 16
    };
    // the request's first factors of this head; those of its other chunks follow at equal distances
    const size_t first = (size_t)c0 * heads + h;
    const size_t spread = (size_t)nc * heads;
    const auto qb = buffer_of(Q + first * CT * DP, spread * CT * DP * 4), kb = buffer_of(KT + first * CT * DP, spread * CT * DP * 4);
    const auto gb = buffer_of(G + first * DP, spread * DP * 4), ab = buffer_of(A + first * CT * CT, spread * CT * CT * 4);
    const int at = 16 * (wave * RL_WAVE + lane), a_at = 4 * (wave * RL_WAVE + lane), decay_at = 4 * (16 * wave + 4 * g);
    // values: the portion's rows from this head's first column on; the last row ends the resource
    const int row_bytes = in.width * (int)sizeof(T);
    const auto vb = buffer_of(in.packed + (size_t)t0 * in.width + in.v_col + h * dv,
                              (size_t)(t1 - t0 - 1) * row_bytes + (size_t)dv * sizeof(T));
    const int tt = threadIdx.x / 16, jj = threadIdx.x % 16;
    const bool column = j0 + jj < dv;
    const int v_at = tt * row_bytes + (j0 + jj) * (int)sizeof(T);
    auto load = [&](int c, Operands& x) {
        const int qc = c * heads * (CT * DP * 4), gc = c * heads * (DP * 4), ac = c * heads * (CT * CT * 4);
#pragma unroll
        for (int m = 0; m < RB; ++m) {
            x.q[m] = load4(qb, at + 4096 * m, qc);
            x.k[m] = load4(kb, at + 4096 * m, qc);
            x.decay[m] = load4(gb, decay_at + 256 * m, gc);
        }
        x.a = load1<float>(ab, a_at, ac);
        x.v = load1<T>(vb, column ? v_at + c * CT * row_bytes : -4, 0);
    };
    // a chunk's values, read by every wave
    auto stage = [&](int c, T raw_value) {
        const float v = to_float(raw_value);
        sv[c & 1][tt][jj] = SILU ? silu<T>(v) : v;
    };
    // the outputs of a chunk: thread (token, column); a column beyond the head is beyond the resource
    const int out_row = heads * dv * 4;
    const auto ob = buffer_of(raw + (size_t)t0 * heads * dv + h * dv, (size_t)(t1 - t0 - 1) * out_row + (size_t)dv * 4);
    const int out_at = tt * out_row + 4 * (j0 + jj);
    auto store = [&](int c) {
        float(*buf)[CT][CT + 1] = red[c & 1];
        const float o = (buf[0][tt][jj] + buf[1][tt][jj]) + (buf[2][tt][jj] + buf[3][tt][jj]);
        __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(o), ob, column ? out_at + c * CT * out_row : -4, 0, 0);
    };
    auto walk = [&](int c, const Operands& x, T next_value, int next, Operands& y, bool more) {
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = sv[c & 1][4 * g + r][r16];
        f32x4 o = (f32x4){0.f, 0.f, 0.f, 0.f};
        // the chunk's own pairs: wave w takes tokens 4g + w
        f32x4 o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a, sv[c & 1][4 * g + wave][r16], o, 0, 0, 0);
#pragma unroll
        for (int m = 0; m < RB; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (r & 1)
                    o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m][r], st[m][r], o2, 0, 0, 0);
                else
                    o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m][r], st[m][r], o, 0, 0, 0);
            }
        if (c > 0) store(c - 1);  // its shares were complete at the last barrier
        if (more) load(next, y);
        stage(c + 1, next_value);
#pragma unroll
        for (int m = 0; m < RB; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) st[m][r] *= x.decay[m][r];
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int m = 0; m < RB; ++m) st[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[m][r], v[r], st[m], 0, 0, 0);
        float(*buf)[CT][CT + 1] = red[c & 1];
#pragma unroll
        for (int r = 0; r < 4; ++r) buf[wave][4 * g + r][r16] = o[r] + o2[r];
        // one barrier a chunk: the other buffer is written next, and this one again only after
        // every wave has passed the next barrier, before which it was read
        __syncthreads();
        __builtin_amdgcn_sched_barrier(0);  // the loads of a chunk stay as far ahead as they are written
    };
    // the operands of the next AHEAD chunks are on their way (they come from memory: the factors were
    // written by workgroups on other XCDs)
    constexpr int BUFS = walk_buffers(RB), AHEAD = BUFS - 1;
    Operands x[BUFS];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) load(min(u, nc - 1), x[u]);
    // Nothing is on its way when the loop is entered: the compiler's waits inside it then stand for the
    // loop's own loads alone.
    __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0)
    stage(0, x[0].v);
    __syncthreads();
    int c = 0;
    for (; c + BUFS <= nc; c += BUFS) {
#pragma unroll
        for (int u = 0; u < BUFS; ++u) walk(c + u, x[u], x[(u + 1) % BUFS].v, min(c + u + AHEAD, nc - 1), x[(u + AHEAD) % BUFS], true);
    }
#pragma unroll
    for (int u = 0; u < AHEAD; ++u)
        if (c + u < nc) walk(c + u, x[u], x[u + 1 < AHEAD ? u + 1 : u].v, 0, x[AHEAD], false);
    store(nc - 1);
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
    return f.sigmoid_gate ? fsigmoid<T>(z) : silu<T>(z);
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
                y.v[e] = from_float<T>(x[e] * rr * (f.sigmoid_gate ? fsigmoid<T>(z) : silu<T>(z)));
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
                y.v[e] = from_float<T>(x[e] * rr * (f.sigmoid_gate ? fsigmoid<T>(z) : silu<T>(z)));
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
    const bool channel = dec.out_t != nullptr;
#define RL_FACTORS(CHANNEL, DP)                                                                                      \
    do {                                                                                                             \
        const size_t lds = sizeof(float) * ((size_t)(CHANNEL ? 4 : 2) * CT * (DP + 4) + 4 * CT * CT +                \
                                            (CHANNEL ? (size_t)CT * ((dec.rank + 3) & ~3) : 0));                     \
        if (lds > 156 * 1024) return RL_ERR_ARG;                                                                     \
        auto kernel = chunk_factors_kernel<T, CHANNEL, DP>;                                                          \
        if (lds > 60 * 1024 &&                                                                                       \
            hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return RL_ERR_LAUNCH;                                                                                    \
        hipLaunchKernelGGL(kernel, dim3(nchunks, heads), dim3(256), lds, stream, in, dec, chunks, Q, KT, G, A, heads, d); \
    } while (0)
#define RL_FACTORS_OF(DP)           \
    do {                            \
        if (channel)                \
            RL_FACTORS(true, DP);   \
        else                        \
            RL_FACTORS(false, DP);  \
    } while (0)
    if (d <= 64)
        RL_FACTORS_OF(64);
    else if (d <= 128)
        RL_FACTORS_OF(128);
    else if (d <= 192)
        RL_FACTORS_OF(192);
    else
        RL_FACTORS_OF(256);
#undef RL_FACTORS_OF
#undef RL_FACTORS
    const int col_groups = (dv + 15) / 16;
    const long groups = ((long)num_seqs * heads * col_groups + XCDS - 1) / XCDS * XCDS;
    if (groups > 0x7fffffffL) return RL_ERR_ARG;
    // a request's factors, values and outputs are addressed by 32-bit offsets (nchunks bounds its chunks)
    const long span = (long)nchunks * CT * ((d + 63) / 64 * 64 > dv ? (d + 63) / 64 * 64 : dv) * heads * 4;
    if (span > 0x7fffff00L || (long)nchunks * CT * in.width * (long)sizeof(T) > 0x7fffff00L) return RL_ERR_ARG;
#define RL_WALK_AS(RB, SILU)                                                                                         \
    hipLaunchKernelGGL((chunk_walk_kernel<T, RB, SILU>), dim3((unsigned)groups), dim3(256), 0, stream, in, Q, KT, G, A, \
                       cu, seq_slots, seq_chunks, S, raw, num_seqs, heads, d, dv, col_groups)
#define RL_WALK(RB)                 \
    do {                            \
        if (in.silu)                \
            RL_WALK_AS(RB, true);   \
        else                        \
            RL_WALK_AS(RB, false);  \
    } while (0)
    if (d <= 64)
        RL_WALK(1);
    else if (d <= 128)
        RL_WALK(2);
    else if (d <= 192)
        RL_WALK(3);
    else
        RL_WALK(4);
#undef RL_WALK_AS
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
// (DP: d up to a multiple of 64) and A [chunks, heads, 256] are scratch.
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
