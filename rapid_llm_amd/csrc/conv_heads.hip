// What attention behind short convolutions reads, from columns of a packed row of the projections,
//   [q: nq * d | k: nkv * d | v: nkv * dv]:
// the projections' bias, a causal convolution over time on every channel (no bias, no activation),
// a norm over the whole of q and the whole of k (all heads together, a weight a channel), the
// rotation of the first channels of every head by the token's position, and the write of the
// queries, and of the keys and values into their pages.  Convolution, norm and rotation are each
// optional; sums, statistics and angles are float32.
//
// The convolution's inputs are the projected values with their bias.  Those before a request's
// first token of the step come from its state rows, [slots][max(taps - 1, 1)][channels] float32,
// oldest first, zeros when the request begins; they are left holding the last taps - 1 inputs
// (by a second launch, after every read; in a step of single tokens by the token's own workgroup).
//
// A workgroup takes the queries and keys of TT consecutive tokens of the flat batch, VEC adjacent
// channels a thread at a time; with TAPS > 0 the inputs that the next token needs again stay in
// registers, and the convolved q and k wait in LDS for their norms.  The values have neither norm
// nor rotation.  In a step of portions (TT = 4) they are further workgroups of the same launch, of 16
// tokens each: four neighbouring threads take four tokens each of the same channels, so that the
// sixteen places of a channel in a page (which are contiguous) are written together.  Cache layout:
// keys [page][nkv][P][d], values [page][nkv][dv][P].
#include "common.h"

namespace conv_heads {

constexpr int MAX_TAPS = 16;

template <typename T, int VEC>
struct alignas(sizeof(T) * VEC) Pack {
    T v[VEC];
};

struct Sizes {
    int width, nq, nkv, d, dv, taps, rotary_half, interleaved, page_size, table_stride;
    float eps;
};

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

constexpr int VALUE_TOKENS = 16;  // of a workgroup of values

template <typename T, int VEC, int TT, int TAPS>
__global__ __launch_bounds__(1024) void prepare_kernel(
    const T* __restrict__ packed, const float* __restrict__ bias, const float* __restrict__ taps_t,
    float* __restrict__ state, const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w,
    const float* __restrict__ cos_tab, const float* __restrict__ sin_tab, T* __restrict__ q_out,
    T* __restrict__ k_cache, T* __restrict__ v_cache, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, const int* __restrict__ cu, int num_seqs,
    int tokens, int single, int qk_groups, Sizes z) {
    extern __shared__ __attribute__((aligned(16))) float conv[];  // [TT][q and k channels]
    constexpr int HELD = TT == 1 ? 1 : VALUE_TOKENS;
    __shared__ int s_offset[HELD], s_slot[HELD], s_pos[HELD], s_page[HELD], s_request[HELD];
    __shared__ float s_sum[2 * TT][16], s_factor[2 * TT];
    const int nqd = z.nq * z.d, qk = nqd + z.nkv * z.d, channels = qk + z.nkv * z.dv;
    const int tid = threadIdx.x, lane = tid & (RL_WAVE - 1), wave = tid / RL_WAVE;
    const bool of_values = TT > 1 && (int)blockIdx.x >= qk_groups;  // (the whole workgroup)
    const int first = of_values ? ((int)blockIdx.x - qk_groups) * VALUE_TOKENS : (int)blockIdx.x * TT;
    const int nt = min(of_values ? VALUE_TOKENS : TT, tokens - first);
    // what is known of each token; of one token alone in registers
    int offset1 = 0, slot1 = 0, pos1 = 0, page1 = 0;
    if constexpr (TT == 1) {
        const int s = single ? first : request_of(cu, num_seqs, first);
        offset1 = single ? 0 : first - cu[s];
        slot1 = token_slot[first];
        pos1 = positions[first];
        page1 = k_cache ? block_table[(size_t)slot1 * z.table_stride + pos1 / z.page_size] : 0;
    } else {
        if (tid < HELD) {
            const int t = min(first + tid, tokens - 1);
            const int s = request_of(cu, num_seqs, t);
            const int pos = positions[t], slot = token_slot[t];
            s_request[tid] = s;
            s_offset[tid] = t - cu[s];
            s_slot[tid] = slot;
            s_pos[tid] = pos;
            s_page[tid] = k_cache ? block_table[(size_t)slot * z.table_stride + pos / z.page_size] : 0;
        }
        __syncthreads();
    }
    auto offset_of = [&](int tt) -> int { return TT == 1 ? offset1 : s_offset[tt]; };
    auto slot_of = [&](int tt) -> int { return TT == 1 ? slot1 : s_slot[tt]; };
    auto pos_of = [&](int tt) -> int { return TT == 1 ? pos1 : s_pos[tt]; };
    auto page_of = [&](int tt) -> int { return TT == 1 ? page1 : s_page[tt]; };
    const int reach = TAPS > 0 ? TAPS : z.taps, held = reach - 1;

    typedef Pack<T, VEC> TP;
    typedef Pack<float, VEC> FP;
    // the projected values (with bias) of token t
    auto projected = [&](int t, int c, const FP& b, float (&u)[VEC]) {
        const TP q = *reinterpret_cast<const TP*>(packed + (size_t)t * z.width + c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = to_float(q.v[e]) + b.v[e];
    };
    // and `back` tokens before the workgroup's token tt
    auto before = [&](int tt, int back, int c, const FP& b, float (&u)[VEC]) {
        const int offset = offset_of(tt);
        if (back <= offset) {
            projected(first + tt - back, c, b, u);
        } else {
            const FP q = *reinterpret_cast<const FP*>(state + ((size_t)slot_of(tt) * held + held + offset - back) * channels + c);
#pragma unroll
            for (int e = 0; e < VEC; ++e) u[e] = q.v[e];
        }
    };
    // the convolved values of channels c .. c + VEC - 1 of the workgroup's tokens tt0 .. tt0 + TT - 1
    auto convolve = [&](int tt0, int c, float (&y)[TT][VEC]) {
        constexpr int WT = TAPS > 0 ? TAPS : 1, WIN = TAPS > 1 ? TAPS - 1 : 1;
        FP wt[WT], b;
        float win[WIN][VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) b.v[e] = 0.f;
        if (bias) b = *reinterpret_cast<const FP*>(bias + c);
        if constexpr (TAPS > 0) {
#pragma unroll
            for (int tap = 0; tap < TAPS; ++tap) wt[tap] = *reinterpret_cast<const FP*>(taps_t + (size_t)tap * channels + c);
        }
#pragma unroll
        for (int n = 0; n < TT; ++n) {
            const int tt = tt0 + n;
            if (tt >= nt) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[n][e] = 0.f;
                continue;
            }
            float now[VEC];
            projected(first + tt, c, b, now);
            if (!taps_t) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[n][e] = now[e];
                continue;
            }
            float acc[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
            float* rows = state + (size_t)slot_of(tt) * max(held, 1) * channels + c;
            if constexpr (TAPS > 0) {
                if (n == 0 || s_request[TT == 1 ? 0 : tt] != s_request[TT == 1 ? 0 : tt - 1]) {
#pragma unroll
                    for (int q = 0; q < TAPS - 1; ++q) before(tt, TAPS - 1 - q, c, b, win[q]);
                }
#pragma unroll
                for (int tap = 0; tap < TAPS - 1; ++tap)
#pragma unroll
                    for (int e = 0; e < VEC; ++e) acc[e] = fmaf(wt[tap].v[e], win[tap][e], acc[e]);
#pragma unroll
                for (int e = 0; e < VEC; ++e) acc[e] = fmaf(wt[TAPS - 1].v[e], now[e], acc[e]);
#pragma unroll
                for (int q = 0; q + 1 < TAPS - 1; ++q)
#pragma unroll
                    for (int e = 0; e < VEC; ++e) win[q][e] = win[q + 1][e];
                if constexpr (TAPS > 1) {
#pragma unroll
                    for (int e = 0; e < VEC; ++e) win[TAPS - 2][e] = now[e];
                    if (single) {
                        // (this thread alone reads these channels of the request's rows)
#pragma unroll
                        for (int q = 0; q < TAPS - 1; ++q) {
                            FP row;
#pragma unroll
                            for (int e = 0; e < VEC; ++e) row.v[e] = win[q][e];
                            *reinterpret_cast<FP*>(rows + (size_t)q * channels) = row;
                        }
                    }
                }
            } else {
                for (int tap = 0; tap < reach; ++tap) {
                    const FP w = *reinterpret_cast<const FP*>(taps_t + (size_t)tap * channels + c);
                    float u[VEC];
                    before(tt, held - tap, c, b, u);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) acc[e] = fmaf(w.v[e], u[e], acc[e]);
                }
                if (single && held > 0) {
                    for (int q = 0; q + 1 < held; ++q)
                        *reinterpret_cast<FP*>(rows + (size_t)q * channels) =
                            *reinterpret_cast<const FP*>(rows + (size_t)(q + 1) * channels);
                    FP last;
#pragma unroll
                    for (int e = 0; e < VEC; ++e) last.v[e] = now[e];
                    *reinterpret_cast<FP*>(rows + (size_t)(held - 1) * channels) = last;
                }
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) y[n][e] = acc[e];
        }
    };
    // channels c .. of the values of tokens tt0 .. into their pages
    auto write_values = [&](int tt0, int c, const float (&y)[TT][VEC]) {
        const int head = c / z.dv, ch = c - head * z.dv;
        auto place = [&](int tt) -> T* {
            return v_cache + (((size_t)page_of(tt) * z.nkv + head) * z.dv + ch) * z.page_size + pos_of(tt) % z.page_size;
        };
        // consecutive places of a page, from a multiple of TT on
        if (TT > 1 && tt0 + TT <= nt && z.page_size % TT == 0 && pos_of(tt0) % TT == 0 &&
            s_request[TT == 1 ? 0 : tt0] == s_request[TT == 1 ? 0 : tt0 + TT - 1]) {
            T* dst = place(tt0);
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                Pack<T, TT> o;
#pragma unroll
                for (int n = 0; n < TT; ++n) o.v[n] = from_float<T>(y[n][e]);
                *reinterpret_cast<Pack<T, TT>*>(dst + (size_t)e * z.page_size) = o;
            }
            return;
        }
#pragma unroll
        for (int n = 0; n < TT; ++n) {
            if (tt0 + n >= nt) continue;
            T* dst = place(tt0 + n);
#pragma unroll
            for (int e = 0; e < VEC; ++e) dst[(size_t)e * z.page_size] = from_float<T>(y[n][e]);
        }
    };

    if constexpr (TT > 1) {
        if (of_values) {
            constexpr int PARTS = VALUE_TOKENS / TT;
            for (int item = tid; item < z.nkv * z.dv / VEC * PARTS; item += blockDim.x) {
                const int tt0 = item % PARTS * TT, c = item / PARTS * VEC;
                if (tt0 >= nt) continue;
                float y[TT][VEC];
                convolve(tt0, qk + c, y);
                write_values(tt0, c, y);
            }
            return;
        }
    }

    // q and k to LDS, with the sums of their squares
    float ss[2][TT];
#pragma unroll
    for (int tt = 0; tt < TT; ++tt) ss[0][tt] = ss[1][tt] = 0.f;
    for (int c = VEC * tid; c < (TT == 1 ? channels : qk); c += VEC * blockDim.x) {
        float y[TT][VEC];
        convolve(0, c, y);
        if (TT == 1 && c >= qk) {
            if (v_cache) write_values(0, c - qk, y);
            continue;
        }
        const bool is_k = c >= nqd;
#pragma unroll
        for (int tt = 0; tt < TT; ++tt) {
            float sq = 0.f;
            FP out;
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                out.v[e] = y[tt][e];
                sq += y[tt][e] * y[tt][e];
            }
            *reinterpret_cast<FP*>(conv + (size_t)tt * qk + c) = out;
            ss[0][tt] += is_k ? 0.f : sq;
            ss[1][tt] += is_k ? sq : 0.f;
        }
    }
    // the norms' sums over the workgroup
#pragma unroll
    for (int n = 0; n < 2 * TT; ++n) {
        const float v = wave_sum(ss[n / TT][n % TT]);
        if (lane == 0) s_sum[n][wave] = v;
    }
    __syncthreads();
    if (tid < 2 * TT) {
        float total = 0.f;
        for (int w = 0; w < (int)blockDim.x / RL_WAVE; ++w) total += s_sum[tid][w];
        s_factor[tid] = rsqrtf(total / (float)(tid < TT ? nqd : qk - nqd) + z.eps);
    }
    __syncthreads();
    for (int c = VEC * tid; c < qk; c += VEC * blockDim.x) {
        const bool is_k = c >= nqd;
        if (is_k ? !k_cache : !q_out) continue;
        const int local = is_k ? c - nqd : c;
        const int head = local / z.d, i = local - head * z.d;
        const float* w = is_k ? k_norm_w : q_norm_w;
        const bool turns = cos_tab && i < 2 * z.rotary_half;
        // whole quads turn with whole quads
        const bool quads = turns && !z.interleaved && z.rotary_half % VEC == 0;
        const bool second = i >= z.rotary_half;
        const int there = second ? -z.rotary_half : z.rotary_half;
        FP weight, weight2;
#pragma unroll
        for (int e = 0; e < VEC; ++e) weight.v[e] = weight2.v[e] = 1.f;
        if (w) {
            weight = *reinterpret_cast<const FP*>(w + local);
            if (quads) weight2 = *reinterpret_cast<const FP*>(w + local + there);
        }
#pragma unroll
        for (int tt = 0; tt < TT; ++tt) {
            if (tt >= nt) continue;
            const float factor = w ? s_factor[is_k ? TT + tt : tt] : 1.f;
            const float* row = conv + (size_t)tt * qk + c;
            const FP own = *reinterpret_cast<const FP*>(row);
            const float* cs = cos_tab + (size_t)pos_of(tt) * z.rotary_half;
            const float* sn = sin_tab + (size_t)pos_of(tt) * z.rotary_half;
            float v[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[e] = own.v[e] * factor * weight.v[e];
            if (quads) {
                const FP other = *reinterpret_cast<const FP*>(row + there);
                const int pair = second ? i - z.rotary_half : i;
                const FP cq = *reinterpret_cast<const FP*>(cs + pair), sq = *reinterpret_cast<const FP*>(sn + pair);
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    const float o = other.v[e] * factor * weight2.v[e];
                    v[e] = second ? v[e] * cq.v[e] + o * sq.v[e] : v[e] * cq.v[e] - o * sq.v[e];
                }
            } else if (turns) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    const int ch = i + e;
                    if (ch >= 2 * z.rotary_half) continue;
                    const bool sec = z.interleaved ? (ch & 1) : ch >= z.rotary_half;
                    const int by = z.interleaved ? 1 : z.rotary_half;
                    const int pair = z.interleaved ? ch >> 1 : (sec ? ch - z.rotary_half : ch);
                    const int at = e + (sec ? -by : by);
                    const float o = row[at] * factor * (w ? w[local + at] : 1.f);
                    v[e] = sec ? v[e] * cs[pair] + o * sn[pair] : v[e] * cs[pair] - o * sn[pair];
                }
            }
            TP out;
#pragma unroll
            for (int e = 0; e < VEC; ++e) out.v[e] = from_float<T>(v[e]);
            T* dst = is_k ? k_cache + (((size_t)page_of(tt) * z.nkv + head) * z.page_size + pos_of(tt) % z.page_size) * z.d + i
                          : q_out + (size_t)(first + tt) * nqd + local;
            *reinterpret_cast<TP*>(dst) = out;
        }
    }
}

// the state rows after a step with portions: the last taps - 1 inputs of every request
template <typename T>
__global__ __launch_bounds__(256) void state_kernel(const T* __restrict__ packed, int width, const float* __restrict__ bias,
                                                    float* __restrict__ state, const int* __restrict__ cu,
                                                    const int* __restrict__ seq_slots, int channels, int taps) {
    const int s = blockIdx.x;
    const int c = blockIdx.y * blockDim.x + threadIdx.x;
    const int held = taps - 1;
    if (c >= channels) return;
    const int t0 = cu[s], n = cu[s + 1] - t0;
    const float b = bias ? bias[c] : 0.f;
    float* st = state + (size_t)seq_slots[s] * held * channels + c;
    // (a row that moves down is read before any later one is written: they go in ascending order)
    for (int q = 0; q < held; ++q) {
        const int rel = n - held + q;  // place in the portion of the input that row q will hold
        st[(size_t)q * channels] = rel >= 0 ? to_float(packed[(size_t)(t0 + rel) * width + c]) + b
                                            : st[(size_t)(q + n) * channels];
    }
}

template <typename T>
static int launch(const T* packed, const float* bias, const float* taps_t, float* state, const float* q_norm_w,
                  const float* k_norm_w, const float* cos_tab, const float* sin_tab, T* q_out, T* k_cache, T* v_cache,
                  const int* positions, const int* token_slot, const int* block_table, const int* cu,
                  const int* seq_slots, int num_seqs, int tokens, const Sizes& z, hipStream_t stream) {
    const int single = tokens == num_seqs;  // every request brings one token
    const int qk = (z.nq + z.nkv) * z.d, channels = qk + z.nkv * z.dv;
    // (the rotation tables' rows are read four entries at a time where whole quads turn)
    const bool vec = z.d % 4 == 0 && z.dv % 4 == 0 && z.width % 4 == 0 && (uintptr_t)packed % (4 * sizeof(T)) == 0;
    const int tt = !single && (size_t)qk * 4 * sizeof(float) <= 80 * 1024 ? 4 : 1;
    const size_t lds = (size_t)tt * qk * sizeof(float);
    if (lds > 156 * 1024) return RL_ERR_ARG;
    const int qk_groups = (tokens + tt - 1) / tt;
    const int value_groups = tt > 1 && v_cache ? (tokens + VALUE_TOKENS - 1) / VALUE_TOKENS : 0;
    const int items = (tt > 1 ? qk : channels) / (vec ? 4 : 1);  // a thread each, where they fit
    dim3 grid(qk_groups + value_groups), block(items >= 1024 ? 1024 : (items + 255) / 256 * 256);
#define RL_HEADS(VEC, TT, TAPS)                                                                                        \
    do {                                                                                                               \
        auto kernel = prepare_kernel<T, VEC, TT, TAPS>;                                                                \
        if (lds > 60 * 1024 &&                                                                                         \
            hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return RL_ERR_LAUNCH;                                                                                      \
        hipLaunchKernelGGL(kernel, grid, block, lds, stream, packed, bias, taps_t, state, q_norm_w, k_norm_w, cos_tab, \
                           sin_tab, q_out, k_cache, v_cache, positions, token_slot, block_table, cu, num_seqs, tokens,  \
                           single, qk_groups, z);                                                                      \
    } while (0)
#define RL_HEADS_TAPS(VEC, TT)                      \
    do {                                            \
        if (taps_t && z.taps == 4)                  \
            RL_HEADS(VEC, TT, 4);                   \
        else                                        \
            RL_HEADS(VEC, TT, 0);                   \
    } while (0)
    if (vec && tt == 4)
        RL_HEADS_TAPS(4, 4);
    else if (vec)
        RL_HEADS_TAPS(4, 1);
    else if (tt == 4)
        RL_HEADS_TAPS(1, 4);
    else
        RL_HEADS_TAPS(1, 1);
#undef RL_HEADS_TAPS
#undef RL_HEADS
    if (taps_t && z.taps > 1 && !single)
        hipLaunchKernelGGL(state_kernel<T>, dim3(num_seqs, (channels + 255) / 256), dim3(256), 0, stream, packed, z.width,
                           bias, state, cu, seq_slots, channels, z.taps);
    return rl_launch_status();
}

}  // namespace conv_heads

extern "C" int rl_conv_heads_max_taps() { return conv_heads::MAX_TAPS; }

// taps_t: [taps][channels] or null (no convolution: no state); norm weights [nq * d] and [nkv * d] or null;
// q_out, k_cache (with v_cache): null where nothing is written there
extern "C" int rl_conv_heads(const void* packed, int width, const float* bias, const float* taps_t, float* state, int taps,
                             const float* q_norm_w, const float* k_norm_w, float eps, const float* cos_tab,
                             const float* sin_tab, int rotary_half, int interleaved, void* q_out, void* k_cache,
                             void* v_cache, const int* positions, const int* token_slot, const int* block_table,
                             int table_stride, int page_size, const int* cu, const int* seq_slots, int num_seqs, int tokens,
                             int nq, int nkv, int d, int dv, int act_type, hipStream_t stream) {
    if (tokens <= 0 || num_seqs <= 0) return RL_OK;
    if (nq < 1 || nkv < 1 || d < 1 || dv < 1 || page_size < 1 || num_seqs > tokens || !k_cache != !v_cache ||
        width < (nq + nkv) * d + nkv * dv || (taps_t && (!state || taps < 1 || taps > conv_heads::MAX_TAPS)) ||
        (cos_tab && (!sin_tab || rotary_half < 1 || 2 * rotary_half > d)))
        return RL_ERR_ARG;
    const conv_heads::Sizes z = {width, nq, nkv, d, dv, taps, rotary_half, interleaved, page_size, table_stride, eps};
    if (act_type == RL_F32)
        return conv_heads::launch<float>((const float*)packed, bias, taps_t, state, q_norm_w, k_norm_w, cos_tab, sin_tab,
                                         (float*)q_out, (float*)k_cache, (float*)v_cache, positions, token_slot,
                                         block_table, cu, seq_slots, num_seqs, tokens, z, stream);
    if (act_type == RL_BF16)
        return conv_heads::launch<bf16_t>((const bf16_t*)packed, bias, taps_t, state, q_norm_w, k_norm_w, cos_tab, sin_tab,
                                          (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, positions, token_slot,
                                          block_table, cu, seq_slots, num_seqs, tokens, z, stream);
    return RL_ERR_ARG;
}
