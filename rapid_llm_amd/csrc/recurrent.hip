// Recurrent mixers with a fixed-size state per request: the token-shift mixes and the per-head
// scan of an RWKV-style time mixing; the causal convolution, the scan and the grouped norm of a
// state-space mixer; the prepared operands and the scan of a gated delta rule with a decay per key
// channel; and a gated recurrence without a matrix state (minGRU).  Everything between the projections is float32: mixes of the decay branch,
// decays, step sizes, states, sums, norms; the element type T only says how the projections'
// results are read and the mixers' outputs written.
//
// A step is a flat batch of requests: request s brings the tokens cu[s] .. cu[s + 1] - 1 and keeps
// its state in row seq_slots[s] of the state tensors.  Every scan walks a request's tokens in
// order with the state in registers, so a token's sums are formed in one order whatever else the
// step holds and however the request's tokens were cut into steps: in float32 the results are
// equal bit for bit.
//
// How a scan is laid out.  A head's state is a matrix [rows i, columns j]; a token multiplies
// every element once or twice and sums over the rows, and the next token cannot start before.
// What bounds a prompt is therefore the time of one token, and that is the state elements a lane
// holds: a wave takes 4 columns and deals the rows to its 16 lanes a column (RPL rows a lane),
// a workgroup of 4 waves takes 16 columns, a head is ceil(columns / 16) workgroups on compute
// units of their own.  The row sums are folded over the 16 lanes by four rotations inside the
// row of lanes (data-parallel primitives, no trip through LDS).  The tokens' operands come
// through LDS sixteen tokens at a time, the next sixteen travelling from memory meanwhile.  The
// state is kept column-major ([j][i]) so that a lane's rows are contiguous.
#include "common.h"

namespace recurrent {

// the request a token of the flat batch belongs to: the last s with cu[s] <= t
__device__ inline int request_of(const int* __restrict__ cu, int num_seqs, int t) {
    int lo = 0, hi = num_seqs - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (cu[mid] <= t)
            lo = mid;
        else
            hi = mid - 1;
    }
    return lo;
}

__device__ inline float silu(float z) { return z / (1.f + expf(-z)); }

// --------------------------------------------------------------------------- //
// Token shift.  With h' the previous token's row (the request's state row before its first token
// of the step), branch b reads h + (h' - h) * mu[b].  Branches 0..3 are written in the compute
// type, side by side as [4][tokens][width]; branch 4 (the decay's) in float32.
// The state row is replaced by the request's last row in a second launch, after every read; in a
// step of single tokens (`single`) a token's workgroup is the only one that touches its request's
// row and replaces it itself.
// --------------------------------------------------------------------------- //
template <typename T>
struct alignas(sizeof(T) * 4) Quad {
    T v[4];
};

template <typename T>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ x, const float* __restrict__ mu,
                                                          float* __restrict__ state, T* __restrict__ mixes,
                                                          float* __restrict__ mix_w, const int* __restrict__ cu,
                                                          const int* __restrict__ seq_slots, int num_seqs,
                                                          int tokens, int width, int single) {
    const int t = blockIdx.x;
    const int s = single ? t : request_of(cu, num_seqs, t);
    const bool first = single || t == cu[s];
    float* prev_state = state + (size_t)seq_slots[s] * width;
    const T* row = x + (size_t)t * width;
    const T* before = x + (size_t)(first ? t : t - 1) * width;
    const size_t plane = (size_t)tokens * width;
    if (width % 4 == 0) {
        // four channels a thread, every access 8 or 16 bytes; the loads of two rounds are asked for together
#pragma unroll 2
        for (int i = 4 * threadIdx.x; i < width; i += 4 * blockDim.x) {
            const Quad<T> hq = *reinterpret_cast<const Quad<T>*>(row + i);
            float p[4];
            if (first) {
                const float4 ps = *reinterpret_cast<const float4*>(prev_state + i);
                p[0] = ps.x; p[1] = ps.y; p[2] = ps.z; p[3] = ps.w;
            } else {
                const Quad<T> pq = *reinterpret_cast<const Quad<T>*>(before + i);
#pragma unroll
                for (int e = 0; e < 4; ++e) p[e] = to_float(pq.v[e]);
            }
            float h[4], d[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                h[e] = to_float(hq.v[e]);
                d[e] = p[e] - h[e];
            }
#pragma unroll
            for (int b = 0; b < 5; ++b) {
                const float4 m = *reinterpret_cast<const float4*>(mu + (size_t)b * width + i);
                const float y[4] = {fmaf(d[0], m.x, h[0]), fmaf(d[1], m.y, h[1]), fmaf(d[2], m.z, h[2]),
                                    fmaf(d[3], m.w, h[3])};
                if (b < 4) {
                    Quad<T> o;
#pragma unroll
                    for (int e = 0; e < 4; ++e) o.v[e] = from_float<T>(y[e]);
                    *reinterpret_cast<Quad<T>*>(mixes + b * plane + (size_t)t * width + i) = o;
                } else {
                    *reinterpret_cast<float4*>(mix_w + (size_t)t * width + i) = make_float4(y[0], y[1], y[2], y[3]);
                }
            }
            if (single) *reinterpret_cast<float4*>(prev_state + i) = make_float4(h[0], h[1], h[2], h[3]);
        }
        return;
    }
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        const float h = to_float(row[i]);
        const float p = first ? prev_state[i] : to_float(before[i]);
        const float d = p - h;
#pragma unroll
        for (int b = 0; b < 4; ++b)
            mixes[b * plane + (size_t)t * width + i] = from_float<T>(fmaf(d, mu[(size_t)b * width + i], h));
        mix_w[(size_t)t * width + i] = fmaf(d, mu[(size_t)4 * width + i], h);
        if (single) prev_state[i] = h;
    }
}

template <typename T>
__global__ __launch_bounds__(256) void shift_state_kernel(const T* __restrict__ x, float* __restrict__ state,
                                                          const int* __restrict__ cu,
                                                          const int* __restrict__ seq_slots, int width) {
    const int s = blockIdx.x;
    const T* last = x + (size_t)(cu[s + 1] - 1) * width;
    float* dst = state + (size_t)seq_slots[s] * width;
    for (int i = threadIdx.x; i < width; i += blockDim.x) dst[i] = to_float(last[i]);
}

// --------------------------------------------------------------------------- //
// Helpers of the scans: the sum over a row of 16 lanes by rotations (every lane gets it; the
// order of the additions is fixed by the lane), and the block of tokens staged in LDS.
// --------------------------------------------------------------------------- //
template <int CTRL>
__device__ inline float ror_add(float v) {
    const int moved = __builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true);
    return v + __int_as_float(moved);
}
__device__ inline float row16_sum(float v) {
    v = ror_add<0x128>(v);  // row_ror:8
    v = ror_add<0x124>(v);  // row_ror:4
    v = ror_add<0x122>(v);  // row_ror:2
    v = ror_add<0x121>(v);  // row_ror:1
    return v;
}
// the same sums for N values at once, one rotation of all of them after the other: a value's four
// additions depend on each other, those of different values do not, and a wave that runs alone on
// its SIMD has nothing else to put between dependent instructions
template <int N>
__device__ inline void row16_sums(float (&v)[N]) {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = ror_add<0x128>(v[i]);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = ror_add<0x124>(v[i]);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = ror_add<0x122>(v[i]);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = ror_add<0x121>(v[i]);
}

// lane + 16's and lane's value, summed in both (every even row of 16 lanes with the odd one behind it)
__device__ inline float both_rows(float v) {
    const unsigned u = __float_as_uint(v);
    const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
    return __uint_as_float(a[0]) + __uint_as_float(a[1]);
}
// the sum over the 16 or 32 lanes of a column, in every one of them
template <int LPC>
__device__ inline float column_sum(float v) {
    v = row16_sum(v);
    if constexpr (LPC == 32) v = both_rows(v);
    return v;
}

// a block's sixteen sums over the lanes of a column: lane c (of 16 or 32) returns token c % 16's
template <int LPC>
__device__ inline float block_sums(float (&os)[16], int c) {
    row16_sums(os);
    // every lane of a row of sixteen holds that row's sums of all tokens: lane c takes token c's,
    // and where a column is two rows of lanes adds the other row's
    float mine = os[0];
#pragma unroll
    for (int tt = 1; tt < 16; ++tt) mine = (c & 15) == tt ? os[tt] : mine;
    if constexpr (LPC == 32) mine = both_rows(mine);
    return mine;
}

// A lane's RPL consecutive state rows from or to memory: sixteen bytes at a time where the rows
// of a column are a multiple of four (a group of four is then wholly inside the column or wholly
// beyond it), else one by one.
template <int RPL>
__device__ inline void state_rows_load(const float* __restrict__ column, int first, int rows, bool live,
                                       float (&state)[RPL]) {
    if constexpr (RPL % 4 == 0) {
        if (rows % 4 == 0) {
#pragma unroll
            for (int q = 0; q < RPL; q += 4) {
                float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
                if (live && first + q < rows) v = *reinterpret_cast<const float4*>(column + first + q);
                state[q] = v.x; state[q + 1] = v.y; state[q + 2] = v.z; state[q + 3] = v.w;
            }
            return;
        }
    }
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii) state[ii] = (live && first + ii < rows) ? column[first + ii] : 0.f;
}
template <int RPL>
__device__ inline void state_rows_store(float* __restrict__ column, int first, int rows, bool live,
                                        const float (&state)[RPL]) {
    if (!live) return;
    if constexpr (RPL % 4 == 0) {
        if (rows % 4 == 0) {
#pragma unroll
            for (int q = 0; q < RPL; q += 4)
                if (first + q < rows)
                    *reinterpret_cast<float4*>(column + first + q) =
                        make_float4(state[q], state[q + 1], state[q + 2], state[q + 3]);
            return;
        }
    }
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii)
        if (first + ii < rows) column[first + ii] = state[ii];
}

// Rows i .. i + 3 of a head of `size` rows: one access where WHOLE (every head starts at a multiple of
// four elements and has a multiple of four rows), else one by one; a row beyond the head is a real
// one that is not used.
template <bool WHOLE, typename T>
__device__ inline Quad<T> load_quad(const T* __restrict__ head, int i, int size) {
    if constexpr (WHOLE) return *reinterpret_cast<const Quad<T>*>(head + min(i, size - 4));
    Quad<T> q;
#pragma unroll
    for (int e = 0; e < 4; ++e) q.v[e] = head[min(i + e, size - 1)];
    return q;
}

constexpr int SCAN_TOKENS = 16;   // tokens staged at a time
constexpr int SCAN_WAVES = 4;                      // waves of a workgroup
// blocks of tokens in LDS at a time: two where three operands of so many rows fit 64 KB twice
constexpr int scan_buffers(int rows) { return rows <= 128 ? 2 : 1; }
// tokens whose operands are read from LDS together, while as many before them are computed (two sets
// of registers: fewer tokens the more rows a lane holds)
constexpr int scan_ahead(int rows) { return rows <= 4 ? 4 : (rows <= 8 ? 2 : 1); }
constexpr int SCAN_THREADS = 64 * SCAN_WAVES;
constexpr int SCAN_COLS = 4 * SCAN_WAVES;          // columns of a workgroup: 4 a wave

// --------------------------------------------------------------------------- //
// The time-mixing scan.  Per head, state S[key channel i][value channel j], kept as [j][i].  For a
// token with r, k, v (d each), the decay w_i = exp(-exp(pre_i + bias_i)), formed as a block of
// tokens is fetched, and the bonus u_i:
//   o_j = sum_i r_i (S_ij + u_i k_i v_j)        S_ij <- w_i S_ij + k_i v_j
// o goes out unfinished (float32); head_finish_kernel divides every head by its root mean square
// and applies the norm's weight and silu(g).
// --------------------------------------------------------------------------- //
// one state element's share of a token (the same instructions wherever a token is computed)
__device__ inline void wkv_row(float r, float k, float w, float u, float vj, float& state, float& o) {
    const float kv = k * vj;
    o = fmaf(r, fmaf(u, kv, state), o);
    state = fmaf(w, state, kv);
}
// the decay exp(-exp(pre + bias)): the library's exponentials in a float32 engine, the hardware's (of base
// 2, in float32) in a bfloat16 one
template <typename T>
__device__ inline float wkv_decay(float pre, float bias) {
    if constexpr (sizeof(T) == 4) return expf(-expf(pre + bias));
    constexpr float log2e = 1.4426950408889634f;
    return __builtin_amdgcn_exp2f(-log2e * __builtin_amdgcn_exp2f(log2e * (pre + bias)));
}

template <typename T, int LPC, int RPL, bool WHOLE>
__global__ __launch_bounds__(SCAN_THREADS) __attribute__((amdgpu_waves_per_eu(1, 2))) void wkv_scan_kernel(
    const T* __restrict__ r, const T* __restrict__ k, const T* __restrict__ v, const float* __restrict__ decay_pre,
    const float* __restrict__ decay_bias, const float* __restrict__ bonus, float* __restrict__ raw,
    const int* __restrict__ cu,
    const int* __restrict__ seq_slots, float* __restrict__ S, int heads, int d) {
    constexpr int DP = LPC * RPL;  // rows, padded
    constexpr int BUFS = scan_buffers(DP);
    constexpr int QUADS = SCAN_TOKENS * DP / 4;  // of a block, four rows of a token each
    constexpr int PER_THREAD = (QUADS + SCAN_THREADS - 1) / SCAN_THREADS;
    constexpr int CPW = RL_WAVE / LPC;      // columns of a wave
    constexpr int COLS = CPW * SCAN_WAVES;  // and of a workgroup
    const int s = blockIdx.x, h = blockIdx.y;
    const int t0 = cu[s], t1 = cu[s + 1];
    const int inner = heads * d;
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = threadIdx.x / RL_WAVE;
    const int c = lane & (LPC - 1);                           // which share of the rows
    const int col = wave * CPW + lane / LPC;                  // column of the workgroup
    const int j = blockIdx.z * COLS + col;
    const bool live = j < d;
    __shared__ __attribute__((aligned(16))) float sr[BUFS][SCAN_TOKENS][DP], sk[BUFS][SCAN_TOKENS][DP],
        sw[BUFS][SCAN_TOKENS][DP];
    __shared__ float sv[BUFS][SCAN_TOKENS][COLS];
    float* Sp = S + (((size_t)seq_slots[s] * heads + h) * d + (live ? j : 0)) * d;
    float state[RPL], u[RPL];
    state_rows_load<RPL>(Sp, c * RPL, d, live, state);
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii) {
        const int i = c * RPL + ii;
        u[ii] = i < d ? bonus[h * d + i] : 0.f;
    }
    // a token's operands from LDS, and this lane's rows' share of its output
    struct Operands {
        float r[RPL], k[RPL], w[RPL], v;
    };
    auto read = [&](int buf, int tt, Operands& x) {
#pragma unroll
        for (int ii = 0; ii < RPL; ++ii) {
            x.r[ii] = sr[buf][tt][c * RPL + ii];
            x.k[ii] = sk[buf][tt][c * RPL + ii];
            x.w[ii] = sw[buf][tt][c * RPL + ii];
        }
        x.v = sv[buf][tt][col];
    };
    auto token = [&](const Operands& x) -> float {
        float o = 0.f;
#pragma unroll
        for (int ii = 0; ii < RPL; ++ii) wkv_row(x.r[ii], x.k[ii], x.w[ii], u[ii], x.v, state[ii], o);
        return o;
    };
    if (t1 - t0 == 1) {
        // a single token: nothing to stage but itself
        const int i = threadIdx.x;
        const size_t at = (size_t)t0 * inner + h * d + i;
        if (i < DP) {
            sr[0][0][i] = i < d ? to_float(r[at]) : 0.f;
            sk[0][0][i] = i < d ? to_float(k[at]) : 0.f;
            sw[0][0][i] = i < d ? wkv_decay<T>(decay_pre[at], decay_bias[h * d + i]) : 0.f;
        }
        const int jj = blockIdx.z * COLS + i;
        if (i < COLS) sv[0][0][i] = jj < d ? to_float(v[(size_t)t0 * inner + h * d + jj]) : 0.f;
        __syncthreads();
        Operands x;
        read(0, 0, x);
        const float o = column_sum<LPC>(token(x));
        if (c == 0 && live) raw[(size_t)t0 * inner + h * d + j] = o;
        state_rows_store<RPL>(Sp, c * RPL, d, live, state);
        return;
    }
    // A block of tokens from memory into registers, as it lies there: quad e of the block's
    // [token][row] arrays.  Nothing is computed from what was asked for until the block is staged
    // (a conversion or an exponential here would wait for the loads where they are issued, and
    // the block before would be computed behind that wait instead of during it), and no load stands
    // behind a condition: beyond the portion or the head a real element is read and not used.
    Quad<T> pr[PER_THREAD], pk[PER_THREAD];
    Quad<float> pw[PER_THREAD], pb[PER_THREAD];
    T pv;
    auto quad_of = [&](int e, int& tt, int& i) {
        const int idx = min(e * SCAN_THREADS + (int)threadIdx.x, QUADS - 1);
        tt = idx / (DP / 4);
        i = 4 * (idx % (DP / 4));
    };
#pragma unroll
    for (int e = 0; e < PER_THREAD; ++e) {
        int tt, i;
        quad_of(e, tt, i);
        pb[e] = load_quad<WHOLE>(decay_bias + h * d, i, d);
    }
    auto fetch = [&](int tb) {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            int tt, i;
            quad_of(e, tt, i);
            const size_t row = (size_t)min(tb + tt, t1 - 1) * inner + h * d;
            pr[e] = load_quad<WHOLE>(r + row, i, d);
            pk[e] = load_quad<WHOLE>(k + row, i, d);
            pw[e] = load_quad<WHOLE>(decay_pre + row, i, d);
        }
        // (threads beyond tokens x columns, where a workgroup has more, carry nothing)
        const int tt = min((int)threadIdx.x / COLS, SCAN_TOKENS - 1), jj = blockIdx.z * COLS + threadIdx.x % COLS;
        pv = v[(size_t)min(tb + tt, t1 - 1) * inner + h * d + min(jj, d - 1)];
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            int tt, i;
            quad_of(e, tt, i);
            float4 rq, kq, wq;
            float* ro = &rq.x;
            float* ko = &kq.x;
            float* wo = &wq.x;
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const bool live_row = i + q < d;
                ro[q] = live_row ? to_float(pr[e].v[q]) : 0.f;
                ko[q] = live_row ? to_float(pk[e].v[q]) : 0.f;
                wo[q] = wkv_decay<T>(pw[e].v[q], pb[e].v[q]);
            }
            *reinterpret_cast<float4*>(&sr[buf][tt][i]) = rq;
            *reinterpret_cast<float4*>(&sk[buf][tt][i]) = kq;
            *reinterpret_cast<float4*>(&sw[buf][tt][i]) = wq;
        }
        if (threadIdx.x < SCAN_TOKENS * COLS) (&sv[buf][0][0])[threadIdx.x] = to_float(pv);
    };
    // With two buffers in LDS the next block is staged, and the one after it asked for, in front of the
    // block at hand: one barrier a block.  With one buffer the waves meet before and after staging.
    // (Beyond the portion real elements are fetched and staged, and not used.)
    int buf = 0;
    fetch(t0);
    if constexpr (BUFS == 2) {
        stage(0);
        fetch(t0 + SCAN_TOKENS);
        __syncthreads();
    }
    for (int tb = t0; tb < t1; tb += SCAN_TOKENS) {
        if constexpr (BUFS == 2) {
            stage(buf ^ 1);
            fetch(tb + 2 * SCAN_TOKENS);
        } else {
            __syncthreads();  // the block before has been read by every wave
            stage(0);
            __syncthreads();
            fetch(tb + SCAN_TOKENS);
        }
        const int nt = min(SCAN_TOKENS, t1 - tb);
        float* dst = raw + (size_t)tb * inner + h * d + j;
        if (nt == SCAN_TOKENS) {
            // a whole block, unrolled and without a branch between its tokens: the reads of later
            // tokens stand in front of the sums of earlier ones, the lane folds of neighbouring
            // tokens interleave, and only the state's own chain orders the tokens; the block's
            // outputs are stored behind it
            // (operands of the next few tokens are read while these are computed)
            constexpr int AHEAD = scan_ahead(RPL);
            float os[SCAN_TOKENS];
            Operands x[2][AHEAD];
#pragma unroll
            for (int q = 0; q < AHEAD; ++q) read(buf, q, x[0][q]);
#pragma unroll
            for (int n = 0; n < SCAN_TOKENS / AHEAD; ++n) {
                if (n + 1 < SCAN_TOKENS / AHEAD) {
#pragma unroll
                    for (int q = 0; q < AHEAD; ++q) read(buf, (n + 1) * AHEAD + q, x[(n + 1) & 1][q]);
                }
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int q = 0; q < AHEAD; ++q) os[n * AHEAD + q] = token(x[n & 1][q]);
            }
            const float mine = block_sums<LPC>(os, c);
            if (live && c < SCAN_TOKENS) dst[(size_t)c * inner] = mine;
        } else {
            for (int tt = 0; tt < nt; ++tt) {
                Operands x;
                read(buf, tt, x);
                const float o = column_sum<LPC>(token(x));
                if (c == 0 && live) dst[(size_t)tt * inner] = o;
            }
        }
        if constexpr (BUFS == 2) {
            buf ^= 1;
            __syncthreads();  // the next block is staged, and this one has been read
        }
    }
    state_rows_store<RPL>(Sp, c * RPL, d, live, state);
}

// out[t, head] = raw / sqrt(mean(raw^2) + eps) * norm_w * gate: one wave a (token, head).  The norm's
// weight has an entry a channel of every head, or (`shared_w`) of one head, for all of them; the gate
// is silu(g) or (`sigmoid_gate`) sigmoid(g).
template <typename T>
__global__ __launch_bounds__(256) void head_finish_kernel(const float* __restrict__ raw, const T* __restrict__ g,
                                                          const float* __restrict__ norm_w, T* __restrict__ out,
                                                          int rows, int heads, int d, float eps, int shared_w,
                                                          int sigmoid_gate) {
    const int row = blockIdx.x * 4 + threadIdx.x / RL_WAVE;  // (token, head)
    const int lane = threadIdx.x & (RL_WAVE - 1);
    if (row >= rows) return;  // whole waves leave
    const size_t base = (size_t)row * d;
    const float* w = norm_w + (shared_w ? 0 : (size_t)(row % heads) * d);
    float ss = 0.f;
    for (int i = lane; i < d; i += RL_WAVE) {
        const float o = raw[base + i];
        ss += o * o;
    }
    const float rr = rsqrtf(wave_sum(ss) / (float)d + eps);
    for (int i = lane; i < d; i += RL_WAVE) {
        const float z = to_float(g[base + i]);
        const float gate = sigmoid_gate ? 1.f / (1.f + expf(-z)) : silu(z);
        out[base + i] = from_float<T>(raw[base + i] * rr * w[i] * gate);
    }
}

// --------------------------------------------------------------------------- //
// Causal convolution per channel over the columns [col0, col0 + channels) of the packed rows, with
// bias and silu: y_t = silu(b + sum_tap w[c][tap] in(t - (taps - 1) + tap)), where inputs before
// the request's first token of the step come from its state rows (the last taps - 1 inputs it has
// seen, oldest first; zeros when the request begins).  A second launch then shifts the state; in a
// step of single tokens (`single`) the thread of a channel shifts its request's rows itself.
// --------------------------------------------------------------------------- //
#define RL_CONV_MAX_TAPS 16

constexpr int CONV_TOKENS = 8;  // consecutive tokens of the flat batch a workgroup takes in a step with portions

template <typename T>
__global__ __launch_bounds__(256) void causal_conv_kernel(const T* __restrict__ packed, int row_width, int col0,
                                                          const float* __restrict__ w, const float* __restrict__ bias,
                                                          float* __restrict__ state, float* __restrict__ out,
                                                          const int* __restrict__ cu,
                                                          const int* __restrict__ seq_slots, int num_seqs, int tokens,
                                                          int channels, int taps, int single, int per_group) {
    const int c = blockIdx.y * blockDim.x + threadIdx.x;
    if (c >= channels) return;
    const int held = taps - 1;
    float wt[RL_CONV_MAX_TAPS];  // this channel's taps
#pragma unroll
    for (int tap = 0; tap < RL_CONV_MAX_TAPS; ++tap) wt[tap] = tap < taps ? w[(size_t)c * taps + tap] : 0.f;
    const float b = bias[c];
    const int first = blockIdx.x * per_group;
    int s = single ? first : request_of(cu, num_seqs, first);
    for (int t = first; t < min(tokens, first + per_group); ++t) {
        if (single)
            s = t;
        else
            while (t >= cu[s + 1]) ++s;  // tokens ascend through the requests
        const int offset = single ? 0 : t - cu[s];  // tokens of the request's portion before this one
        float* st = state + (size_t)seq_slots[s] * max(held, 1) * channels;
        float acc = b;
#pragma unroll
        for (int tap = 0; tap < RL_CONV_MAX_TAPS; ++tap) {
            if (tap < taps) {
                const int rel = offset - held + tap;  // offset in the portion of the input this tap meets
                const float in = rel >= 0 ? to_float(packed[(size_t)(t - offset + rel) * row_width + col0 + c])
                                          : st[(size_t)(held + rel) * channels + c];
                acc = fmaf(wt[tap], in, acc);
            }
        }
        out[(size_t)t * channels + c] = silu(acc);
        if (single && held > 0) {
            for (int q = 0; q + 1 < held; ++q) st[(size_t)q * channels + c] = st[(size_t)(q + 1) * channels + c];
            st[(size_t)(held - 1) * channels + c] = to_float(packed[(size_t)t * row_width + col0 + c]);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void conv_state_kernel(const T* __restrict__ packed, int row_width, int col0,
                                                         float* __restrict__ state, const int* __restrict__ cu,
                                                         const int* __restrict__ seq_slots, int channels, int taps) {
    const int s = blockIdx.x;
    const int c = blockIdx.y * blockDim.x + threadIdx.x;
    const int held = taps - 1;
    if (c >= channels || held < 1) return;
    const int t0 = cu[s], n = cu[s + 1] - cu[s];
    float* st = state + (size_t)seq_slots[s] * held * channels;
    float old[RL_CONV_MAX_TAPS];
#pragma unroll
    for (int q = 0; q < RL_CONV_MAX_TAPS; ++q) old[q] = q < held ? st[(size_t)q * channels + c] : 0.f;
#pragma unroll
    for (int q = 0; q < RL_CONV_MAX_TAPS; ++q) {
        if (q >= held) continue;
        const int rel = n - held + q;
        float value = 0.f;
        if (rel >= 0) {
            value = to_float(packed[(size_t)(t0 + rel) * row_width + col0 + c]);
        } else {
#pragma unroll
            for (int z = 0; z < RL_CONV_MAX_TAPS; ++z)
                if (z == q + n) value = old[z];
        }
        st[(size_t)q * channels + c] = value;
    }
}

// --------------------------------------------------------------------------- //
// The state-space scan.  `mixed` rows are [x: heads * P | B: groups * N | C: groups * N] (float32,
// behind convolution and silu); per head, state S[n][p], kept as [p][n].  As a block of tokens is
// fetched the raw step sizes become dt = softplus(dt_raw + dt_bias) and a = exp(-exp(A_log) dt); then
//   S_np <- a S_np + dt B_n x_p          y_p = sum_n S_np C_n + D x_p
// and y_p silu(z_p) is written (z: the first heads * P columns of the packed rows).
// --------------------------------------------------------------------------- //
__device__ inline float ssm_step_size(float raw, float bias) {
    const float pre = raw + bias;
    return pre > 20.f ? pre : log1pf(expf(pre));
}
__device__ inline float ssm_decay(float a_log, float dt) { return expf(-expf(a_log) * dt); }
// one state element's share of a token, and the finished output of a channel
__device__ inline void ssm_row(float a, float B, float C, float dx, float& state, float& y) {
    state = fmaf(B, dx, a * state);
    y = fmaf(state, C, y);
}
__device__ inline float ssm_out(float y, float D, float x, float z) { return fmaf(D, x, y) * silu(z); }

template <typename T, int RPL>
__global__ __launch_bounds__(SCAN_THREADS) __attribute__((amdgpu_waves_per_eu(1, 2))) void ssm_scan_kernel(
    const float* __restrict__ mixed, const float* __restrict__ dt_raw, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const float* __restrict__ skip, const T* __restrict__ packed, int row_width, float* __restrict__ out, const int* __restrict__ cu,
    const int* __restrict__ seq_slots, float* __restrict__ S, int heads, int P, int N, int groups) {
    constexpr int NP = 16 * RPL;  // state rows, padded
    constexpr int PER_THREAD = SCAN_TOKENS * NP / SCAN_THREADS;  // = RPL
    const int s = blockIdx.x, h = blockIdx.y;
    const int t0 = cu[s], t1 = cu[s + 1];
    const int inner = heads * P;
    const int channels = inner + 2 * groups * N;
    const int grp = h / (heads / groups);
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = threadIdx.x / RL_WAVE;
    const int c = lane & 15;
    const int col = wave * 4 + (lane >> 4);
    const int p = blockIdx.z * SCAN_COLS + col;
    const bool live = p < P;
    __shared__ __attribute__((aligned(16))) float sB[SCAN_TOKENS][NP], sC[SCAN_TOKENS][NP];
    __shared__ float sx[SCAN_TOKENS][SCAN_COLS], sz[SCAN_TOKENS][SCAN_COLS], sdt[SCAN_TOKENS], sa[SCAN_TOKENS];
    float* Sp = S + (((size_t)seq_slots[s] * heads + h) * P + (live ? p : 0)) * N;
    float state[RPL];
    state_rows_load<RPL>(Sp, c * RPL, N, live, state);
    const float D = skip[h];
    // a block of tokens from memory into registers as it lies there; step sizes and decays are
    // formed when the block is staged, not where its loads are issued
    float pB[PER_THREAD], pC[PER_THREAD], px = 0.f, pd = 0.f;
    T pz = from_float<T>(0.f);
    const float step_bias = dt_bias[h], rate_log = a_log[h];
    auto fetch = [&](int tb) {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            const int idx = e * SCAN_THREADS + threadIdx.x;
            const int tt = idx / NP, n = idx % NP;
            const bool ok = tb + tt < t1 && n < N;
            const float* row = mixed + (size_t)(tb + tt) * channels + inner + grp * N + n;
            pB[e] = ok ? row[0] : 0.f;
            pC[e] = ok ? row[groups * N] : 0.f;
        }
        const int tt = threadIdx.x / SCAN_COLS, pp = blockIdx.z * SCAN_COLS + threadIdx.x % SCAN_COLS;
        const bool ok = tt < SCAN_TOKENS && tb + tt < t1 && pp < P;
        px = ok ? mixed[(size_t)(tb + tt) * channels + h * P + pp] : 0.f;
        pz = ok ? packed[(size_t)(tb + tt) * row_width + h * P + pp] : from_float<T>(0.f);
        // threads 0..15 carry the step sizes, threads 16..31 the decays of the block's tokens
        const int tk = threadIdx.x & 15;
        pd = (threadIdx.x < 32 && tb + tk < t1) ? dt_raw[(size_t)(tb + tk) * heads + h] : 0.f;
    };
    auto stage = [&]() {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            const int idx = e * SCAN_THREADS + threadIdx.x;
            (&sB[0][0])[idx] = pB[e];
            (&sC[0][0])[idx] = pC[e];
        }
        if (threadIdx.x < SCAN_TOKENS * SCAN_COLS) {
            (&sx[0][0])[threadIdx.x] = px;
            (&sz[0][0])[threadIdx.x] = to_float(pz);
        }
        if (threadIdx.x < 32) {
            const float dt = ssm_step_size(pd, step_bias);
            if (threadIdx.x < 16) sdt[threadIdx.x] = dt;
            else sa[threadIdx.x - 16] = ssm_decay(rate_log, dt);
        }
    };
    fetch(t0);
    for (int tb = t0; tb < t1; tb += SCAN_TOKENS) {
        __syncthreads();  // the block before has been read by every wave
        stage();
        __syncthreads();
        if (tb + SCAN_TOKENS < t1) fetch(tb + SCAN_TOKENS);
        const int nt = min(SCAN_TOKENS, t1 - tb);
        auto token = [&](int tt) -> float {
            const float x = sx[tt][col], a = sa[tt];
            const float dx = sdt[tt] * x;
            float y = 0.f;
#pragma unroll
            for (int ii = 0; ii < RPL; ++ii)
                ssm_row(a, sB[tt][c * RPL + ii], sC[tt][c * RPL + ii], dx, state[ii], y);
            return y;  // this lane's rows' share
        };
        float* dst = out + (size_t)tb * inner + h * P + p;
        if (nt == SCAN_TOKENS) {
            // a whole block without a branch between its tokens
            float ys[SCAN_TOKENS];
#pragma unroll
            for (int tt = 0; tt < SCAN_TOKENS; ++tt) ys[tt] = token(tt);
            row16_sums(ys);
            // every lane of a column holds all sixteen sums: lane c finishes and stores token c's
            // (skip term, gate with its exponential and division: once a lane, not once a token)
            float mine = ys[0];
#pragma unroll
            for (int tt = 1; tt < SCAN_TOKENS; ++tt) mine = c == tt ? ys[tt] : mine;
            if (live) dst[(size_t)c * inner] = ssm_out(mine, D, sx[c][col], sz[c][col]);
        } else {
            for (int tt = 0; tt < nt; ++tt) {
                const float y = row16_sum(token(tt));
                if (c == 0 && live) dst[(size_t)tt * inner] = ssm_out(y, D, sx[tt][col], sz[tt][col]);
            }
        }
    }
    state_rows_store<RPL>(Sp, c * RPL, N, live, state);
}

// out[t, part] = y[t, part] / sqrt(mean(y[t, part]^2) + eps) * w, a row in `parts` equal parts
template <typename T>
__global__ __launch_bounds__(256) void group_rmsnorm_kernel(const float* __restrict__ y, const float* __restrict__ w,
                                                            T* __restrict__ out, int width, int parts, float eps) {
    __shared__ float scratch[16];
    const int size = width / parts;
    const size_t base = (size_t)blockIdx.x * width + (size_t)blockIdx.y * size;
    float ss = 0.f;
    for (int i = threadIdx.x; i < size; i += blockDim.x) {
        const float v = y[base + i];
        ss += v * v;
    }
    ss = block_sum(ss, scratch);
    const float rr = rsqrtf(ss / (float)size + eps);
    for (int i = threadIdx.x; i < size; i += blockDim.x)
        out[base + i] = from_float<T>(y[base + i] * rr * w[blockIdx.y * size + i]);
}

// --------------------------------------------------------------------------- //
// Gated delta rule with a decay per key channel.  The packed rows hold, from column col0 on,
// [q: kv_heads * d | k: kv_heads * d | v: heads * dv]; every channel passes a causal convolution over
// time (the state rows before a request's first token, as above) and silu; then every head of q and k
// is made a unit vector (x / sqrt(sum x^2 + 1e-6)) and q is multiplied by d^(-1/2).  The decays'
// pre-activations become g = exp(-exp(A_log_h) softplus(pre + dt_bias)) in place.
//
// One wave takes one head of q, k, v or of the decays for per_group consecutive tokens of the flat
// batch, EPL adjacent channels a lane; with TAPS > 0 the inputs of the last TAPS - 1 tokens stay in
// its registers, so that an input is read once.  In a step of single tokens (`single`) the wave
// shifts its request's convolution rows itself, otherwise conv_state_kernel does in a second launch.
// --------------------------------------------------------------------------- //
constexpr float UNIT_EPS = 1e-6f;
constexpr int PREPARE_TOKENS = 8;

__device__ inline float softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

template <typename T, int TAPS, int EPL>
__global__ __launch_bounds__(256) void delta_prepare_kernel(
    const T* __restrict__ packed, int row_width, int col0, const float* __restrict__ w, float* __restrict__ state,
    float* __restrict__ decay, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
    float* __restrict__ mixed, const int* __restrict__ cu, const int* __restrict__ seq_slots, int num_seqs, int tokens,
    int heads, int kv_heads, int d, int dv, int taps, int single, int per_group) {
    const int head = blockIdx.y * 4 + threadIdx.x / RL_WAVE;
    const int lane = threadIdx.x & (RL_WAVE - 1);
    const int convolved = 2 * kv_heads + heads;
    if (head >= convolved + heads) return;  // whole waves leave; no barrier follows
    const int first = blockIdx.x * per_group, last = min(tokens, first + per_group);
    if (head >= convolved) {
        const int h = head - convolved;
        const float rate = expf(a_log[h]);
        for (int t = first; t < last; ++t)
#pragma unroll
            for (int e = 0; e < EPL; ++e) {
                const int i = lane * EPL + e;
                if (i >= d) continue;
                float* at = decay + (size_t)t * heads * d + h * d + i;
                *at = expf(-rate * softplus(*at + dt_bias[h * d + i]));
            }
        return;
    }
    const bool is_v = head >= 2 * kv_heads, is_q = head < kv_heads;
    const int size = is_v ? dv : d;
    const int c0 = is_v ? 2 * kv_heads * d + (head - 2 * kv_heads) * dv : head * d;  // of the convolved channels
    const int channels = 2 * kv_heads * d + heads * dv;
    const int reach = TAPS > 0 ? TAPS : taps;
    const int held = reach - 1;
    constexpr int WT = TAPS > 0 ? TAPS : 1, WIN = TAPS > 1 ? TAPS - 1 : 1;
    float wt[EPL][WT], win[EPL][WIN];
    if constexpr (TAPS > 0) {
#pragma unroll
        for (int e = 0; e < EPL; ++e)
#pragma unroll
            for (int tap = 0; tap < TAPS; ++tap)
                wt[e][tap] = lane * EPL + e < size ? w[(size_t)(c0 + lane * EPL + e) * TAPS + tap] : 0.f;
    }
    int s = single ? first : request_of(cu, num_seqs, first);
    const float* st = nullptr;
    // what the channel at `c` met `back` tokens before token t, the offset-th of its portion
    auto input = [&](int t, int offset, int back, int c) -> float {
        return back <= offset ? to_float(packed[(size_t)(t - back) * row_width + col0 + c])
                              : st[(size_t)(held + offset - back) * channels + c];
    };
    bool fresh = true;  // the window does not hold the tokens before this one yet
    for (int t = first; t < last; ++t) {
        if (single) {
            s = t;
            fresh = true;
        } else {
            while (t >= cu[s + 1]) {  // tokens ascend through the requests
                ++s;
                fresh = true;
            }
        }
        const int offset = single ? 0 : t - cu[s];
        if (fresh) st = state + (size_t)seq_slots[s] * max(held, 1) * channels;
        float y[EPL], now[EPL];
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < EPL; ++e) {
            const int i = lane * EPL + e, c = c0 + i;
            const bool live = i < size;
            now[e] = live ? to_float(packed[(size_t)t * row_width + col0 + c]) : 0.f;
            float acc = 0.f;
            if constexpr (TAPS > 0) {
                if (fresh) {
#pragma unroll
                    for (int q = 0; q < TAPS - 1; ++q) win[e][q] = live ? input(t, offset, TAPS - 1 - q, c) : 0.f;
                }
#pragma unroll
                for (int tap = 0; tap < TAPS - 1; ++tap) acc = fmaf(wt[e][tap], win[e][tap], acc);
                acc = fmaf(wt[e][TAPS - 1], now[e], acc);
            } else if (live) {
                for (int tap = 0; tap < held; ++tap)
                    acc = fmaf(w[(size_t)c * reach + tap], input(t, offset, held - tap, c), acc);
                acc = fmaf(w[(size_t)c * reach + held], now[e], acc);
            }
            y[e] = live ? silu(acc) : 0.f;
            ss += y[e] * y[e];
        }
        float factor = 1.f;
        if (!is_v) {
            factor = rsqrtf(wave_sum(ss) + UNIT_EPS);
            if (is_q) factor *= rsqrtf((float)d);
        }
        float* dst = mixed + (size_t)t * channels + c0;
#pragma unroll
        for (int e = 0; e < EPL; ++e) {
            const int i = lane * EPL + e;
            if (i < size) dst[i] = y[e] * factor;
            if (single && held > 0 && i < size) {
                float* rows = state + (size_t)seq_slots[s] * held * channels + c0 + i;
                for (int q = 0; q + 1 < held; ++q) rows[(size_t)q * channels] = rows[(size_t)(q + 1) * channels];
                rows[(size_t)(held - 1) * channels] = now[e];
            }
            if constexpr (TAPS > 1) {
#pragma unroll
                for (int q = 0; q + 1 < TAPS - 1; ++q) win[e][q] = win[e][q + 1];
                win[e][TAPS - 2] = now[e];
            }
        }
        fresh = false;
    }
}

// The scan.  Per head (head h reads q and k of kv head h / (heads / kv_heads)), state S[key channel i]
// [value channel j], kept as [j][i]; for a token with q, k, v, the decays g and beta = sigmoid(b):
//   S_ij <- g_i S_ij      u_j = beta (v_j - sum_i S_ij k_i)      S_ij <- S_ij + k_i u_j      o_j = sum_i S_ij q_i
// The sum that u needs stands between two tokens and is folded at once; the read-out's sums are folded
// behind a block of tokens.  o goes out unfinished (float32).
template <int LPC, int RPL, bool WHOLE>
__global__ __launch_bounds__(SCAN_THREADS) __attribute__((amdgpu_waves_per_eu(1, 2))) void delta_scan_kernel(
    const float* __restrict__ mixed, const float* __restrict__ decay, const float* __restrict__ beta_pre,
    int beta_width, float* __restrict__ raw, const int* __restrict__ cu, const int* __restrict__ seq_slots,
    float* __restrict__ S, int heads, int kv_heads, int d, int dv) {
    constexpr int DP = LPC * RPL;  // rows, padded
    constexpr int BUFS = scan_buffers(DP);
    constexpr int QUADS = SCAN_TOKENS * DP / 4;  // of a block, four rows of a token each
    constexpr int PER_THREAD = (QUADS + SCAN_THREADS - 1) / SCAN_THREADS;
    constexpr int CPW = RL_WAVE / LPC;       // columns of a wave
    constexpr int COLS = CPW * SCAN_WAVES;   // and of a workgroup
    const int s = blockIdx.x, h = blockIdx.y;
    const int t0 = cu[s], t1 = cu[s + 1];
    const int channels = 2 * kv_heads * d + heads * dv;
    const int hk = h / (heads / kv_heads);
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = threadIdx.x / RL_WAVE;
    const int c = lane & (LPC - 1);
    const int col = wave * CPW + lane / LPC;
    const int j = blockIdx.z * COLS + col;
    const bool live = j < dv;
    __shared__ __attribute__((aligned(16))) float sq[BUFS][SCAN_TOKENS][DP], sk[BUFS][SCAN_TOKENS][DP],
        sg[BUFS][SCAN_TOKENS][DP];
    __shared__ float sv[BUFS][SCAN_TOKENS][COLS], sb[BUFS][SCAN_TOKENS];
    float* Sp = S + (((size_t)seq_slots[s] * heads + h) * dv + (live ? j : 0)) * d;
    float state[RPL];
    state_rows_load<RPL>(Sp, c * RPL, d, live, state);
    // a token's operands from LDS, and this lane's rows' share of its output
    struct Operands {
        float q[RPL], k[RPL], g[RPL], v, beta;
    };
    auto read = [&](int buf, int tt, Operands& x) {
#pragma unroll
        for (int ii = 0; ii < RPL; ++ii) {
            x.q[ii] = sq[buf][tt][c * RPL + ii];
            x.k[ii] = sk[buf][tt][c * RPL + ii];
            x.g[ii] = sg[buf][tt][c * RPL + ii];
        }
        x.v = sv[buf][tt][col];
        x.beta = sb[buf][tt];
    };
    auto token = [&](const Operands& x) -> float {
        float even = 0.f, odd = 0.f;
#pragma unroll
        for (int ii = 0; ii < RPL; ++ii) {
            state[ii] *= x.g[ii];
            float& sum = (ii & 1) ? odd : even;
            sum = fmaf(state[ii], x.k[ii], sum);
        }
        const float u = x.beta * (x.v - column_sum<LPC>(even + odd));
        float o = 0.f;
#pragma unroll
        for (int ii = 0; ii < RPL; ++ii) {
            state[ii] = fmaf(x.k[ii], u, state[ii]);
            o = fmaf(state[ii], x.q[ii], o);
        }
        return o;
    };
    if (t1 - t0 == 1) {
        // a single token: nothing to stage but itself
        const int i = threadIdx.x;
        const float* row = mixed + (size_t)t0 * channels;
        if (i < DP) {
            sq[0][0][i] = i < d ? row[hk * d + i] : 0.f;
            sk[0][0][i] = i < d ? row[(kv_heads + hk) * d + i] : 0.f;
            sg[0][0][i] = i < d ? decay[(size_t)t0 * heads * d + h * d + i] : 0.f;
        }
        const int jj = blockIdx.z * COLS + i;
        if (i < COLS) sv[0][0][i] = jj < dv ? row[2 * kv_heads * d + h * dv + jj] : 0.f;
        if (i == 0) sb[0][0] = 1.f / (1.f + expf(-beta_pre[(size_t)t0 * beta_width + h]));
        __syncthreads();
        Operands x;
        read(0, 0, x);
        const float o = column_sum<LPC>(token(x));
        if (c == 0 && live) raw[(size_t)t0 * heads * dv + h * dv + j] = o;
        state_rows_store<RPL>(Sp, c * RPL, d, live, state);
        return;
    }
    // a block of tokens from memory into registers, as the time mixing's
    Quad<float> pq[PER_THREAD], pk[PER_THREAD], pg[PER_THREAD];
    float pv, pb;
    auto quad_of = [&](int e, int& tt, int& i) {
        const int idx = min(e * SCAN_THREADS + (int)threadIdx.x, QUADS - 1);
        tt = idx / (DP / 4);
        i = 4 * (idx % (DP / 4));
    };
    auto fetch = [&](int tb) {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            int tt, i;
            quad_of(e, tt, i);
            const size_t t = min(tb + tt, t1 - 1);
            pq[e] = load_quad<WHOLE>(mixed + t * channels + hk * d, i, d);
            pk[e] = load_quad<WHOLE>(mixed + t * channels + (kv_heads + hk) * d, i, d);
            pg[e] = load_quad<WHOLE>(decay + (t * heads + h) * d, i, d);
        }
        const int tt = min((int)threadIdx.x / COLS, SCAN_TOKENS - 1), jj = blockIdx.z * COLS + threadIdx.x % COLS;
        pv = mixed[(size_t)min(tb + tt, t1 - 1) * channels + 2 * kv_heads * d + h * dv + min(jj, dv - 1)];
        pb = beta_pre[(size_t)min(tb + ((int)threadIdx.x & (SCAN_TOKENS - 1)), t1 - 1) * beta_width + h];
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int e = 0; e < PER_THREAD; ++e) {
            int tt, i;
            quad_of(e, tt, i);
            float4 qq, kq;
            float* qo = &qq.x;
            float* ko = &kq.x;
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                qo[q] = i + q < d ? pq[e].v[q] : 0.f;
                ko[q] = i + q < d ? pk[e].v[q] : 0.f;
            }
            *reinterpret_cast<float4*>(&sq[buf][tt][i]) = qq;
            *reinterpret_cast<float4*>(&sk[buf][tt][i]) = kq;
            *reinterpret_cast<Quad<float>*>(&sg[buf][tt][i]) = pg[e];
        }
        if (threadIdx.x < SCAN_TOKENS * COLS) (&sv[buf][0][0])[threadIdx.x] = pv;
        if (threadIdx.x < SCAN_TOKENS) sb[buf][threadIdx.x] = 1.f / (1.f + expf(-pb));
    };
    // With two buffers in LDS the next block is staged, and the one after it asked for, in front of the
    // block at hand: one barrier a block.  With one buffer the waves meet before and after staging.
    // (Beyond the portion real elements are fetched and staged, and not used.)
    int buf = 0;
    fetch(t0);
    if constexpr (BUFS == 2) {
        stage(0);
        fetch(t0 + SCAN_TOKENS);
        __syncthreads();
    }
    for (int tb = t0; tb < t1; tb += SCAN_TOKENS) {
        if constexpr (BUFS == 2) {
            stage(buf ^ 1);
            fetch(tb + 2 * SCAN_TOKENS);
        } else {
            __syncthreads();  // the block before has been read by every wave
            stage(0);
            __syncthreads();
            fetch(tb + SCAN_TOKENS);
        }
        const int nt = min(SCAN_TOKENS, t1 - tb);
        float* dst = raw + (size_t)tb * heads * dv + h * dv + j;
        if (nt == SCAN_TOKENS) {
            constexpr int AHEAD = scan_ahead(RPL);
            float os[SCAN_TOKENS];
            Operands x[2][AHEAD];
#pragma unroll
            for (int q = 0; q < AHEAD; ++q) read(buf, q, x[0][q]);
#pragma unroll
            for (int n = 0; n < SCAN_TOKENS / AHEAD; ++n) {
                if (n + 1 < SCAN_TOKENS / AHEAD) {
#pragma unroll
                    for (int q = 0; q < AHEAD; ++q) read(buf, (n + 1) * AHEAD + q, x[(n + 1) & 1][q]);
                }
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int q = 0; q < AHEAD; ++q) os[n * AHEAD + q] = token(x[n & 1][q]);
            }
            const float mine = block_sums<LPC>(os, c);
            if (live && c < SCAN_TOKENS) dst[(size_t)c * heads * dv] = mine;
        } else {
            for (int tt = 0; tt < nt; ++tt) {
                Operands x;
                read(buf, tt, x);
                const float o = column_sum<LPC>(token(x));
                if (c == 0 && live) dst[(size_t)tt * heads * dv] = o;
            }
        }
        if constexpr (BUFS == 2) {
            buf ^= 1;
            __syncthreads();  // the next block is staged, and this one has been read
        }
    }
    state_rows_store<RPL>(Sp, c * RPL, d, live, state);
}

// --------------------------------------------------------------------------- //
// Gated recurrence whose gates read the current token alone (minGRU).  With z = sigmoid(zp + bz) and
// u = xp + bx of the packed row's columns z0 and x0 on, per channel
//   S <- (1 - z) S + z (u >= 0 ? u + 1/2 : sigmoid(u))        out = scale * S * silu(gp)
// The chain between tokens is one fused multiply-add, everything else is independent of it.  A
// workgroup takes 8 channels and 64 tokens at a time in three stages that run side by side: four
// waves form the two factors of block i and finish the outputs of block i - 2, while lanes of the
// first wave walk the chain of block i - 1; the stages meet in LDS, one barrier a block.
// --------------------------------------------------------------------------- //
constexpr int GRU_CHANNELS = 8;
constexpr int GRU_TOKENS = 64;
constexpr int XCDS = 8;
constexpr int GRU_WORKERS = 256;                   // threads behind the first wave
constexpr int GRU_PITCH = GRU_TOKENS + 4;          // a channel's tokens side by side

// float32 keeps the library's exponential and division, bfloat16 takes the hardware's instructions
template <typename T>
__device__ inline float sigmoid_of(float x);
template <>
__device__ inline float sigmoid_of<float>(float x) {
    return 1.f / (1.f + expf(-x));
}
template <>
__device__ inline float sigmoid_of<bf16_t>(float x) {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}

// the two factors of the chain
template <typename T>
__device__ inline void gru_factors(float zp, float u, float& keep, float& add) {
    const float z = sigmoid_of<T>(zp);
    const float candidate = u >= 0.f ? u + 0.5f : sigmoid_of<T>(u);
    keep = 1.f - z;
    add = z * candidate;
}

template <typename T>
__global__ __launch_bounds__(RL_WAVE + GRU_WORKERS) void gru_scan_kernel(
    const T* __restrict__ packed, int row_width, int z0, int x0, int g0, const float* __restrict__ bz,
    const float* __restrict__ bx, float* __restrict__ S, T* __restrict__ out, int out_width, float scale,
    const int* __restrict__ cu, const int* __restrict__ seq_slots, int width, int num_seqs, int channel_blocks) {
    constexpr int PER = GRU_TOKENS * GRU_CHANNELS / GRU_WORKERS;  // elements of a block a worker takes
    constexpr int APART = GRU_WORKERS / GRU_CHANNELS;             // tokens between them
    // Workgroups go to the chip's XCDs in turn, each with an L2 of its own, and a memory line holds the
    // channels of several workgroups: neighbouring channels are dealt to the same XCD.
    const int per_xcd = gridDim.x / XCDS;  // (the launch is a multiple)
    const int work = (blockIdx.x % XCDS) * per_xcd + blockIdx.x / XCDS;
    if (work >= num_seqs * channel_blocks) return;  // whole workgroups leave
    const int s = work / channel_blocks;
    const int t0 = cu[s], t1 = cu[s + 1];
    const bool walks = threadIdx.x < RL_WAVE;
    const int w = walks ? threadIdx.x : threadIdx.x - RL_WAVE;
    const int ch = w % GRU_CHANNELS, tt0 = w / GRU_CHANNELS;
    const int c = (work % channel_blocks) * GRU_CHANNELS + ch;
    const bool live = c < width;
    __shared__ __attribute__((aligned(16))) float keep[2][GRU_CHANNELS][GRU_PITCH], add[2][GRU_CHANNELS][GRU_PITCH],
        sums[2][GRU_CHANNELS][GRU_PITCH];
    const float zb = live ? bz[c] : 0.f, xb = live ? bx[c] : 0.f;
    float* slot = S + (size_t)seq_slots[s] * width + c;
    const bool chain = walks && w < GRU_CHANNELS && live;
    float state = chain ? *slot : 0.f;
    T pz[PER], px[PER], pg[PER];
    // (no load stands behind a condition: beyond the portion or the channels a real element is read
    // and not used)
    const T* column = packed + min(c, width - 1);
    auto fetch = [&](int block) {
#pragma unroll
        for (int e = 0; e < PER; ++e) {
            const T* row = column + (size_t)min(t0 + block * GRU_TOKENS + tt0 + e * APART, t1 - 1) * row_width;
            pz[e] = row[z0];
            px[e] = row[x0];
            pg[e] = row[g0];
        }
    };
    const int blocks = (t1 - t0 + GRU_TOKENS - 1) / GRU_TOKENS;
    float gate[PER], gate1[PER], gate2[PER];  // of the block at hand and of the two before it
#pragma unroll
    for (int e = 0; e < PER; ++e) gate[e] = gate1[e] = gate2[e] = 0.f;
    if (!walks) fetch(0);
    for (int i = 0; i < blocks + 2; ++i) {
        if (walks) {
            if (chain && i >= 1 && i <= blocks) {
                const float4* k4 = reinterpret_cast<const float4*>(keep[(i - 1) & 1][ch]);
                const float4* a4 = reinterpret_cast<const float4*>(add[(i - 1) & 1][ch]);
                float4* s4 = reinterpret_cast<float4*>(sums[(i - 1) & 1][ch]);
                // sixteen tokens' factors are asked for while the sixteen before them are walked
                constexpr int BATCH = 4, BATCHES = GRU_TOKENS / 4 / BATCH;
                float4 k[2][BATCH], a[2][BATCH];
#pragma unroll
                for (int q = 0; q < BATCH; ++q) {
                    k[0][q] = k4[q];
                    a[0][q] = a4[q];
                }
#pragma unroll
                for (int n = 0; n < BATCHES; ++n) {
                    if (n + 1 < BATCHES) {
#pragma unroll
                        for (int q = 0; q < BATCH; ++q) {
                            k[(n + 1) & 1][q] = k4[(n + 1) * BATCH + q];
                            a[(n + 1) & 1][q] = a4[(n + 1) * BATCH + q];
                        }
                    }
                    __builtin_amdgcn_sched_barrier(0);  // the reads stay in front of the chain
#pragma unroll
                    for (int q = 0; q < BATCH; ++q) {
                        const float4 kk = k[n & 1][q], aa = a[n & 1][q];
                        float4 o;
                        o.x = state = fmaf(kk.x, state, aa.x);
                        o.y = state = fmaf(kk.y, state, aa.y);
                        o.z = state = fmaf(kk.z, state, aa.z);
                        o.w = state = fmaf(kk.w, state, aa.w);
                        s4[n * BATCH + q] = o;
                    }
                }
            }
        } else {
#pragma unroll
            for (int e = 0; e < PER; ++e) {
                gate2[e] = gate1[e];
                gate1[e] = gate[e];
            }
            float zs[PER], xs[PER], gs[PER];
#pragma unroll
            for (int e = 0; e < PER; ++e) {
                zs[e] = to_float(pz[e]) + zb;
                xs[e] = to_float(px[e]) + xb;
                gs[e] = to_float(pg[e]);
            }
            fetch(i + 1);
            __builtin_amdgcn_sched_barrier(0);  // the next block travels while this one is computed
#pragma unroll
            for (int e = 0; e < PER; ++e) {
                const int tt = tt0 + e * APART;
                float k, a;
                gru_factors<T>(zs[e], xs[e], k, a);
                const bool ok = t0 + i * GRU_TOKENS + tt < t1;  // beyond the portion the state stays as it is
                keep[i & 1][ch][tt] = ok ? k : 1.f;
                add[i & 1][ch][tt] = ok ? a : 0.f;
                gate[e] = scale * gs[e] * sigmoid_of<T>(gs[e]);
            }
            if (i >= 2) {
#pragma unroll
                for (int e = 0; e < PER; ++e) {
                    const int tt = tt0 + e * APART, t = t0 + (i - 2) * GRU_TOKENS + tt;
                    if (live && t < t1) out[(size_t)t * out_width + c] = from_float<T>(gate2[e] * sums[i & 1][ch][tt]);
                }
            }
        }
        __syncthreads();
    }
    if (chain) *slot = state;
}

// a step of single tokens: one thread a (request, channel)
template <typename T>
__global__ __launch_bounds__(256) void gru_single_kernel(const T* __restrict__ packed, int row_width, int z0, int x0,
                                                         int g0, const float* __restrict__ bz,
                                                         const float* __restrict__ bx, float* __restrict__ S,
                                                         T* __restrict__ out, int out_width, float scale,
                                                         const int* __restrict__ seq_slots, int width) {
    const int t = blockIdx.x;  // the request's only token
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= width) return;
    const T* row = packed + (size_t)t * row_width + c;
    float* slot = S + (size_t)seq_slots[t] * width + c;
    float keep, add;
    gru_factors<T>(to_float(row[z0]) + bz[c], to_float(row[x0]) + bx[c], keep, add);
    const float state = fmaf(keep, *slot, add);
    *slot = state;
    const float z = to_float(row[g0]);
    const float gate = scale * z * sigmoid_of<T>(z);
    out[(size_t)t * out_width + c] = from_float<T>(gate * state);
}

}  // namespace recurrent

extern "C" int rl_recurrent_max_head_dim() { return 256; }
extern "C" int rl_conv_max_taps() { return RL_CONV_MAX_TAPS; }

extern "C" int rl_token_shift(const void* x, const float* mu, float* state, void* mixes, float* mix_w,
                              const int* cu, const int* seq_slots, int num_seqs, int tokens, int width,
                              int act_type, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (width < 1) return RL_ERR_ARG;
    const int single = tokens == num_seqs;  // every request brings one token
    if (act_type == RL_F32) {
        hipLaunchKernelGGL(recurrent::token_shift_kernel<float>, dim3(tokens), dim3(256), 0, stream, (const float*)x,
                           mu, state, (float*)mixes, mix_w, cu, seq_slots, num_seqs, tokens, width, single);
        if (!single)
            hipLaunchKernelGGL(recurrent::shift_state_kernel<float>, dim3(num_seqs), dim3(256), 0, stream,
                           (const float*)x, state, cu, seq_slots, width);
    } else if (act_type == RL_BF16) {
        hipLaunchKernelGGL(recurrent::token_shift_kernel<bf16_t>, dim3(tokens), dim3(256), 0, stream,
                           (const bf16_t*)x, mu, state, (bf16_t*)mixes, mix_w, cu, seq_slots, num_seqs, tokens,
                           width, single);
        if (!single)
            hipLaunchKernelGGL(recurrent::shift_state_kernel<bf16_t>, dim3(num_seqs), dim3(256), 0, stream,
                           (const bf16_t*)x, state, cu, seq_slots, width);
    } else {
        return RL_ERR_ARG;
    }
    return rl_launch_status();
}

template <typename T>
static int launch_wkv(const T* r, const T* k, const T* v, const T* g, const float* decay, const float* decay_bias,
                      const float* bonus, const float* norm_w, T* out, float* raw, const int* cu,
                      const int* seq_slots, float* S, int num_seqs, int tokens, int heads, int d, float eps,
                      hipStream_t stream) {
#define RL_WKV_AS(LPC, RPL, WHOLE)                                                                                  \
    hipLaunchKernelGGL((recurrent::wkv_scan_kernel<T, LPC, RPL, WHOLE>), dim3(num_seqs, heads, (d + cols - 1) / cols), \
                       dim3(recurrent::SCAN_THREADS), 0, stream, r, k, v, decay, decay_bias, bonus, raw, cu,        \
                       seq_slots, S, heads, d)
#define RL_WKV(LPC, RPL)                                           \
    do {                                                           \
        constexpr int cols = RL_WAVE / LPC * recurrent::SCAN_WAVES; \
        if (d % 4 == 0)                                            \
            RL_WKV_AS(LPC, RPL, true);                             \
        else                                                       \
            RL_WKV_AS(LPC, RPL, false);                            \
    } while (0)
    // Two rows of lanes a column where one row's workgroups of one request leave half the chip or more
    // without one.  (A property of the model, not of the step: a token's sums keep one order.)
    const bool wide = heads * ((d + 15) / 16) <= 128;
    if (d <= 16)
        RL_WKV(16, 1);
    else if (d <= 32)
        RL_WKV(16, 2);
    else if (d <= 64) {
        if (wide)
            RL_WKV(32, 2);
        else
            RL_WKV(16, 4);
    } else if (d <= 128) {
        if (wide)
            RL_WKV(32, 4);
        else
            RL_WKV(16, 8);
    } else if (wide)
        RL_WKV(32, 8);
    else
        RL_WKV(16, 16);
#undef RL_WKV
#undef RL_WKV_AS
    const int heads_rows = tokens * heads;
    hipLaunchKernelGGL(recurrent::head_finish_kernel<T>, dim3((heads_rows + 3) / 4), dim3(256), 0, stream, raw, g,
                       norm_w, out, heads_rows, heads, d, eps, 0, 0);
    return rl_launch_status();
}

// decay: the decays' pre-activations [tokens, heads * d]; raw: [tokens, heads * d] float32 scratch
// for the unfinished outputs
extern "C" int rl_wkv_scan(const void* r, const void* k, const void* v, const void* g, const float* decay,
                           const float* decay_bias, const float* bonus, const float* norm_w, void* out,
                           float* raw, const int* cu, const int* seq_slots, float* S, int num_seqs, int tokens,
                           int heads, int d, float eps, int act_type, hipStream_t stream) {
    if (num_seqs <= 0 || tokens <= 0) return RL_OK;
    if (heads < 1 || heads > 65535 || d < 1 || d > 256 || num_seqs > 65535) return RL_ERR_ARG;
    if (act_type == RL_F32)
        return launch_wkv<float>((const float*)r, (const float*)k, (const float*)v, (const float*)g, decay,
                                 decay_bias, bonus, norm_w, (float*)out, raw, cu, seq_slots, S, num_seqs, tokens,
                                 heads, d, eps, stream);
    if (act_type == RL_BF16)
        return launch_wkv<bf16_t>((const bf16_t*)r, (const bf16_t*)k, (const bf16_t*)v, (const bf16_t*)g, decay,
                                  decay_bias, bonus, norm_w, (bf16_t*)out, raw, cu, seq_slots, S, num_seqs, tokens,
                                  heads, d, eps, stream);
    return RL_ERR_ARG;
}

extern "C" int rl_causal_conv(const void* packed, int row_width, int col0, const float* w, const float* bias,
                              float* state, float* out, const int* cu, const int* seq_slots, int num_seqs,
                              int tokens, int channels, int taps, int act_type, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (channels < 1 || taps < 1 || taps > RL_CONV_MAX_TAPS || col0 < 0 || col0 + channels > row_width)
        return RL_ERR_ARG;
    const int cblocks = (channels + 255) / 256;
    const int single = tokens == num_seqs;  // every request brings one token
    if (cblocks > 65535) return RL_ERR_ARG;
    // single tokens: a workgroup a token, so that no token waits for another
    const int per_group = single ? 1 : recurrent::CONV_TOKENS;
    dim3 grid((tokens + per_group - 1) / per_group, cblocks), sgrid(num_seqs, cblocks);
    if (act_type == RL_F32) {
        hipLaunchKernelGGL(recurrent::causal_conv_kernel<float>, grid, dim3(256), 0, stream, (const float*)packed,
                           row_width, col0, w, bias, state, out, cu, seq_slots, num_seqs, tokens, channels, taps, single, per_group);
        if (taps > 1 && !single)
            hipLaunchKernelGGL(recurrent::conv_state_kernel<float>, sgrid, dim3(256), 0, stream,
                               (const float*)packed, row_width, col0, state, cu, seq_slots, channels, taps);
    } else if (act_type == RL_BF16) {
        hipLaunchKernelGGL(recurrent::causal_conv_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)packed,
                           row_width, col0, w, bias, state, out, cu, seq_slots, num_seqs, tokens, channels, taps, single, per_group);
        if (taps > 1 && !single)
            hipLaunchKernelGGL(recurrent::conv_state_kernel<bf16_t>, sgrid, dim3(256), 0, stream,
                               (const bf16_t*)packed, row_width, col0, state, cu, seq_slots, channels, taps);
    } else {
        return RL_ERR_ARG;
    }
    return rl_launch_status();
}

template <typename T>
static int launch_ssm(const float* mixed, const float* dt_raw, const float* dt_bias, const float* a_log,
                      const float* skip, const T* packed, int row_width, float* out, const int* cu,
                      const int* seq_slots, float* S, int num_seqs, int tokens, int heads, int P, int N, int groups,
                      hipStream_t stream) {
    dim3 grid(num_seqs, heads, (P + recurrent::SCAN_COLS - 1) / recurrent::SCAN_COLS);
#define RL_SSM(RPL)                                                                                           \
    hipLaunchKernelGGL((recurrent::ssm_scan_kernel<T, RPL>), grid, dim3(recurrent::SCAN_THREADS), 0, stream, mixed, \
                       dt_raw, dt_bias, a_log, skip, packed, row_width, out, cu, seq_slots, S, heads, P, N, groups)
    const int rows = (N + 15) / 16;
    if (rows <= 1)
        RL_SSM(1);
    else if (rows <= 2)
        RL_SSM(2);
    else if (rows <= 4)
        RL_SSM(4);
    else if (rows <= 8)
        RL_SSM(8);
    else
        RL_SSM(16);
#undef RL_SSM
    return rl_launch_status();
}

extern "C" int rl_ssm_scan(const float* mixed, const float* dt_raw, const float* dt_bias, const float* a_log,
                           const float* skip, const void* packed, int row_width, float* out,
                           const int* cu, const int* seq_slots, float* S, int num_seqs, int tokens, int heads, int P,
                           int N, int groups, int act_type, hipStream_t stream) {
    if (num_seqs <= 0 || tokens <= 0) return RL_OK;
    if (heads < 1 || heads > 65535 || groups < 1 || heads % groups || P < 1 || P > 256 || N < 1 || N > 256 ||
        row_width < heads * P || num_seqs > 65535)
        return RL_ERR_ARG;
    if (act_type == RL_F32)
        return launch_ssm<float>(mixed, dt_raw, dt_bias, a_log, skip, (const float*)packed, row_width, out, cu,
                                 seq_slots, S, num_seqs, tokens, heads, P, N, groups, stream);
    if (act_type == RL_BF16)
        return launch_ssm<bf16_t>(mixed, dt_raw, dt_bias, a_log, skip, (const bf16_t*)packed, row_width, out,
                                  cu, seq_slots, S, num_seqs, tokens, heads, P, N, groups, stream);
    return RL_ERR_ARG;
}

extern "C" int rl_group_rmsnorm(const float* y, const float* w, void* out, int tokens, int width, int parts,
                                float eps, int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (width < 1 || parts < 1 || width % parts || parts > 65535) return RL_ERR_ARG;
    dim3 grid(tokens, parts);
    if (act_type == RL_F32)
        hipLaunchKernelGGL(recurrent::group_rmsnorm_kernel<float>, grid, dim3(256), 0, stream, y, w, (float*)out,
                           width, parts, eps);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(recurrent::group_rmsnorm_kernel<bf16_t>, grid, dim3(256), 0, stream, y, w, (bf16_t*)out,
                           width, parts, eps);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

template <typename T, int TAPS, int EPL>
static void launch_delta_prepare(const T* packed, int row_width, int col0, const float* w, float* state, float* decay,
                                 const float* dt_bias, const float* a_log, float* mixed, const int* cu,
                                 const int* seq_slots, int num_seqs, int tokens, int heads, int kv_heads, int d, int dv,
                                 int taps, hipStream_t stream) {
    const int single = tokens == num_seqs;  // every request brings one token
    const int per_group = single ? 1 : recurrent::PREPARE_TOKENS;
    dim3 grid((tokens + per_group - 1) / per_group, (2 * kv_heads + 2 * heads + 3) / 4);
    hipLaunchKernelGGL((recurrent::delta_prepare_kernel<T, TAPS, EPL>), grid, dim3(256), 0, stream, packed, row_width,
                       col0, w, state, decay, dt_bias, a_log, mixed, cu, seq_slots, num_seqs, tokens, heads, kv_heads,
                       d, dv, taps, single, per_group);
    if (!single && taps > 1) {
        const int channels = 2 * kv_heads * d + heads * dv;
        hipLaunchKernelGGL(recurrent::conv_state_kernel<T>, dim3(num_seqs, (channels + 255) / 256), dim3(256), 0, stream,
                           packed, row_width, col0, state, cu, seq_slots, channels, taps);
    }
}

template <typename T>
static int delta_prepare(const T* packed, int row_width, int col0, const float* w, float* state, float* decay,
                         const float* dt_bias, const float* a_log, float* mixed, const int* cu, const int* seq_slots,
                         int num_seqs, int tokens, int heads, int kv_heads, int d, int dv, int taps,
                         hipStream_t stream) {
    const int widest = d > dv ? d : dv;
#define RL_PREPARE(TAPS, EPL)                                                                                        \
    launch_delta_prepare<T, TAPS, EPL>(packed, row_width, col0, w, state, decay, dt_bias, a_log, mixed, cu, seq_slots, \
                                       num_seqs, tokens, heads, kv_heads, d, dv, taps, stream)
#define RL_PREPARE_TAPS(TAPS)         \
    do {                              \
        if (widest <= 64)             \
            RL_PREPARE(TAPS, 1);      \
        else if (widest <= 128)       \
            RL_PREPARE(TAPS, 2);      \
        else                          \
            RL_PREPARE(TAPS, 4);      \
    } while (0)
    if (taps == 4)
        RL_PREPARE_TAPS(4);
    else
        RL_PREPARE_TAPS(0);
#undef RL_PREPARE_TAPS
#undef RL_PREPARE
    return rl_launch_status();
}

// decay: the decays' pre-activations [tokens, heads * d], replaced by the decays; mixed:
// [tokens, 2 * kv_heads * d + heads * dv] float32
extern "C" int rl_delta_prepare(const void* packed, int row_width, int col0, const float* w, float* state,
                                float* decay, const float* dt_bias, const float* a_log, float* mixed, const int* cu,
                                const int* seq_slots, int num_seqs, int tokens, int heads, int kv_heads, int d, int dv,
                                int taps, int act_type, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (heads < 1 || kv_heads < 1 || heads % kv_heads || heads > 65535 || d < 1 || d > 256 || dv < 1 || dv > 256 ||
        taps < 1 || taps > RL_CONV_MAX_TAPS || col0 < 0 || col0 + 2 * kv_heads * d + heads * dv > row_width ||
        num_seqs > tokens)
        return RL_ERR_ARG;
    if (act_type == RL_F32)
        return delta_prepare<float>((const float*)packed, row_width, col0, w, state, decay, dt_bias, a_log, mixed, cu,
                                    seq_slots, num_seqs, tokens, heads, kv_heads, d, dv, taps, stream);
    if (act_type == RL_BF16)
        return delta_prepare<bf16_t>((const bf16_t*)packed, row_width, col0, w, state, decay, dt_bias, a_log, mixed, cu,
                                     seq_slots, num_seqs, tokens, heads, kv_heads, d, dv, taps, stream);
    return RL_ERR_ARG;
}

// beta_pre: a float32 row of beta_width a token whose first `heads` entries are the pre-activations;
// raw: [tokens, heads * dv] float32
extern "C" int rl_delta_scan(const float* mixed, const float* decay, const float* beta_pre, int beta_width, float* raw,
                             const int* cu, const int* seq_slots, float* S, int num_seqs, int tokens, int heads,
                             int kv_heads, int d, int dv, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (heads < 1 || heads > 65535 || kv_heads < 1 || heads % kv_heads || d < 1 || d > 256 || dv < 1 || dv > 256 ||
        beta_width < heads || num_seqs > 65535)
        return RL_ERR_ARG;
#define RL_DELTA_AS(LPC, RPL, WHOLE)                                                                                  \
    hipLaunchKernelGGL((recurrent::delta_scan_kernel<LPC, RPL, WHOLE>), dim3(num_seqs, heads, (dv + cols - 1) / cols), \
                       dim3(recurrent::SCAN_THREADS), 0, stream, mixed, decay, beta_pre, beta_width, raw, cu,         \
                       seq_slots, S, heads, kv_heads, d, dv)
#define RL_DELTA(LPC, RPL)                                         \
    do {                                                           \
        constexpr int cols = RL_WAVE / LPC * recurrent::SCAN_WAVES; \
        if (d % 4 == 0 && dv % 4 == 0)                             \
            RL_DELTA_AS(LPC, RPL, true);                           \
        else                                                       \
            RL_DELTA_AS(LPC, RPL, false);                          \
    } while (0)
    const bool wide = heads * ((dv + 15) / 16) <= 256;  // as for the time mixing
    if (d <= 16)
        RL_DELTA(16, 1);
    else if (d <= 32)
        RL_DELTA(16, 2);
    else if (d <= 64) {
        if (wide)
            RL_DELTA(32, 2);
        else
            RL_DELTA(16, 4);
    } else if (d <= 128) {
        if (wide)
            RL_DELTA(32, 4);
        else
            RL_DELTA(16, 8);
    } else if (wide)
        RL_DELTA(32, 8);
    else
        RL_DELTA(16, 16);
#undef RL_DELTA
#undef RL_DELTA_AS
    return rl_launch_status();
}

// raw, g and out: [tokens, heads * d]; norm_w: [heads * d], or [d] with shared_w
extern "C" int rl_head_finish(const float* raw, const void* g, const float* norm_w, void* out, int tokens, int heads,
                              int d, float eps, int shared_w, int sigmoid_gate, int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (heads < 1 || d < 1) return RL_ERR_ARG;
    const int rows = tokens * heads;
    if (act_type == RL_F32)
        hipLaunchKernelGGL(recurrent::head_finish_kernel<float>, dim3((rows + 3) / 4), dim3(256), 0, stream, raw,
                           (const float*)g, norm_w, (float*)out, rows, heads, d, eps, shared_w, sigmoid_gate);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(recurrent::head_finish_kernel<bf16_t>, dim3((rows + 3) / 4), dim3(256), 0, stream, raw,
                           (const bf16_t*)g, norm_w, (bf16_t*)out, rows, heads, d, eps, shared_w, sigmoid_gate);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

template <typename T>
static int launch_gru(const T* packed, int row_width, int z0, int x0, int g0, const float* bz, const float* bx,
                      float* S, T* out, int out_width, float scale, const int* cu, const int* seq_slots, int num_seqs,
                      int tokens, int width, hipStream_t stream) {
    if (tokens == num_seqs)  // every request brings one token
        hipLaunchKernelGGL(recurrent::gru_single_kernel<T>, dim3(tokens, (width + 255) / 256), dim3(256), 0, stream,
                           packed, row_width, z0, x0, g0, bz, bx, S, out, out_width, scale, seq_slots, width);
    else {
        const int blocks = (width + recurrent::GRU_CHANNELS - 1) / recurrent::GRU_CHANNELS;
        const long groups = ((long)num_seqs * blocks + recurrent::XCDS - 1) / recurrent::XCDS * recurrent::XCDS;
        if (groups > 0x7fffffffL) return RL_ERR_ARG;
        hipLaunchKernelGGL(recurrent::gru_scan_kernel<T>, dim3((unsigned)groups),
                           dim3(RL_WAVE + recurrent::GRU_WORKERS), 0, stream, packed, row_width, z0, x0, g0, bz, bx, S,
                           out, out_width, scale, cu, seq_slots, width, num_seqs, blocks);
    }
    return rl_launch_status();
}

// out: the first of `width` columns of rows of out_width elements
extern "C" int rl_gru_scan(const void* packed, int row_width, int z0, int x0, int g0, const float* bz, const float* bx,
                           float* S, void* out, int out_width, float scale, const int* cu, const int* seq_slots,
                           int num_seqs, int tokens, int width, int act_type, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (width < 1 || width > 65535 * recurrent::GRU_CHANNELS || out_width < width || num_seqs > tokens) return RL_ERR_ARG;
    for (int col : {z0, x0, g0})
        if (col < 0 || col + width > row_width) return RL_ERR_ARG;
    if (act_type == RL_F32)
        return launch_gru<float>((const float*)packed, row_width, z0, x0, g0, bz, bx, S, (float*)out, out_width, scale,
                                 cu, seq_slots, num_seqs, tokens, width, stream);
    if (act_type == RL_BF16)
        return launch_gru<bf16_t>((const bf16_t*)packed, row_width, z0, x0, g0, bz, bx, S, (bf16_t*)out, out_width,
                                  scale, cu, seq_slots, num_seqs, tokens, width, stream);
    return RL_ERR_ARG;
}
