// Router of a mixture whose experts are chosen by corrected scores, with experts that return their
// input and a gate for a shared expert, in one kernel, float32 throughout:
//   z = W x over `experts` experts with tensors, `identity` experts without, and, with `gate`, one more row;
//   s = softmax(z) over the experts + identity; chosen: the `top` largest s + correction (the lower
//   index wins a tie); a chosen expert's weight is s * scale (not divided by anything).
// A token's row of `out` has experts + 2 entries: the experts' weights (0 for those not chosen), the
// sigmoid of the gate's row (1 without one), and the sum of the chosen identity experts' weights.
//
// A workgroup takes 16 tokens.  The product runs on the true 32-bit matrix instruction
// (v_mfma_f32_16x16x4_f32) or, where x and W are both bfloat16, on the bfloat16 one
// (v_mfma_f32_16x16x32_bf16: a product of two bfloat16 numbers is exact in float32, and the sums are
// float32 in either), its inner dimension dealt to 16 waves in steps of 16 or 32; their shares are
// added in the order of the waves, so a token's logits do not depend on what else is in the step.
// Then every wave takes a token and chooses.
#include "common.h"

namespace router {

constexpr int TOKENS = 16;
constexpr int WAVES = 16;
constexpr int BLOCKS = 2;  // of 16 rows of W, multiplied with what is read of x
constexpr int MAX_CHOICES = 1024;
typedef float f32x4 __attribute__((ext_vector_type(4)));

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

// what a lane reads of a row at a time: four elements, or eight where both operands are bfloat16
template <typename T, int N>
struct alignas(sizeof(T) * N) Pack {
    T v[N];
};

// acc[16 x 16] += A[16 x 4 packs] B[4 packs x 16]
template <typename T>
__device__ inline f32x4 mma(const Pack<T, 4>& a, const Pack<float, 4>& b, f32x4 acc) {
#pragma unroll
    for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(to_float(a.v[e]), b.v[e], acc, 0, 0, 0);
    return acc;
}
__device__ inline f32x4 mma(const Pack<bf16_t, 8>& a, const Pack<bf16_t, 8>& b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
}

// maximum and sum over a wave, in every lane: four rotations within the rows of 16 lanes, two swaps of rows
template <int CTRL>
__device__ inline float rotated(float v) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
template <typename F>
__device__ inline float over_wave(float v, F f) {
    v = f(v, rotated<0x128>(v));
    v = f(v, rotated<0x124>(v));
    v = f(v, rotated<0x122>(v));
    v = f(v, rotated<0x121>(v));
    const unsigned u = __float_as_uint(v);
    const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
    const unsigned w = __float_as_uint(f(__uint_as_float(a[0]), __uint_as_float(a[1])));
    const auto b = __builtin_amdgcn_permlane32_swap(w, w, false, false);
    return f(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ inline float max_over_wave(float v) {
    return over_wave(v, [](float a, float b) { return fmaxf(a, b); });
}
__device__ inline float sum_over_wave(float v) {
    return over_wave(v, [](float a, float b) { return a + b; });
}

// elements i .. i + N - 1 of a row of k; WHOLE: they are all there (k is a multiple of a step)
template <bool WHOLE, int N, typename T>
__device__ inline Pack<T, N> pack_at(const T* __restrict__ row, int i, int k) {
    if constexpr (WHOLE) return *reinterpret_cast<const Pack<T, N>*>(row + i);
    Pack<T, N> q;
#pragma unroll
    for (int e = 0; e < N; ++e) q.v[e] = i + e < k ? row[i + e] : from_float<T>(0.f);
    return q;
}

template <typename T, typename W, bool WHOLE, int PER>
__global__ __launch_bounds__(WAVES* RL_WAVE) void choose_experts_kernel(
    const T* __restrict__ x, const W* __restrict__ w, const float* __restrict__ correction, float* __restrict__ out,
    int tokens, int k, int experts, int identity, int gate, int top, float scale) {
    constexpr int N = sizeof(W) == 2 ? 8 : 4;  // elements of a lane
    constexpr int STEP = 4 * N;                // and of the four lanes of a row
    extern __shared__ float s_logits[];  // [TOKENS][pitch]
    __shared__ float red[BLOCKS][WAVES][16][17];
    const int choices = experts + identity, rows = choices + gate;
    const int row_blocks = (rows + 15) / 16;
    const int pitch = (row_blocks + BLOCKS - 1) / BLOCKS * BLOCKS * 16 + 1;
    const int tid = threadIdx.x, lane = tid & (RL_WAVE - 1), wave = tid / RL_WAVE;
    const int r16 = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * TOKENS;
    const T* xr = x + (size_t)min(t0 + r16, tokens - 1) * k;
    for (int b0 = 0; b0 < row_blocks; b0 += BLOCKS) {
        f32x4 acc[BLOCKS];
        const W* wr[BLOCKS];
#pragma unroll
        for (int b = 0; b < BLOCKS; ++b) {
            acc[b] = (f32x4){0.f, 0.f, 0.f, 0.f};
            wr[b] = w + (size_t)min(16 * (b0 + b) + r16, rows - 1) * k;  // (beyond the rows: a real one, not used)
        }
        // four steps' operands are asked for together (a step of a few tokens is all latency here)
        for (int i0 = STEP * wave; i0 < k; i0 += 4 * STEP * WAVES) {
            Pack<T, N> xq[4];
            Pack<W, N> wq[4][BLOCKS];
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int i = i0 + q * STEP * WAVES;
                const int at = (i < k ? i : i0) + N * g;  // (beyond the row: the first step's again, not used)
                xq[q] = pack_at<WHOLE, N>(xr, at, k);
#pragma unroll
                for (int b = 0; b < BLOCKS; ++b) wq[q][b] = pack_at<WHOLE, N>(wr[b], at, k);
            }
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                if (i0 + q * STEP * WAVES >= k) continue;
#pragma unroll
                for (int b = 0; b < BLOCKS; ++b) acc[b] = mma(xq[q], wq[q][b], acc[b]);
            }
        }
#pragma unroll
        for (int b = 0; b < BLOCKS; ++b)
#pragma unroll
            for (int e = 0; e < 4; ++e) red[b][wave][4 * g + e][r16] = acc[b][e];
        __syncthreads();
        if (tid < BLOCKS * 256) {
            const int b = tid / 256, t = (tid / 16) % 16, e = tid % 16;
            float sum = 0.f;
#pragma unroll
            for (int v = 0; v < WAVES; ++v) sum += red[b][v][t][e];
            s_logits[t * pitch + 16 * (b0 + b) + e] = sum;
        }
        __syncthreads();
    }
    const int t = t0 + wave;
    if (t >= tokens) return;  // whole waves leave; no barrier follows
    const float* z = s_logits + wave * pitch;
    float s[PER];
    float m = -INFINITY;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
        const int e = lane + RL_WAVE * p;
        s[p] = e < choices ? z[e] : -INFINITY;
        m = fmaxf(m, s[p]);
    }
    m = max_over_wave(m);
    float total = 0.f;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
        s[p] = expf(s[p] - m);
        total += s[p];
    }
    total = sum_over_wave(total);
    float choice[PER];
#pragma unroll
    for (int p = 0; p < PER; ++p) {
        const int e = lane + RL_WAVE * p;
        s[p] /= total;
        choice[p] = e < choices ? s[p] + (correction ? correction[e] : 0.f) : -INFINITY;
    }
    unsigned taken = 0;
    for (int n = 0; n < top; ++n) {
        float best = -INFINITY;
#pragma unroll
        for (int p = 0; p < PER; ++p) best = fmaxf(best, (taken >> p & 1) ? -INFINITY : choice[p]);
        best = max_over_wave(best);
        // the first expert that has it
        bool found = false;
#pragma unroll
        for (int p = 0; p < PER; ++p) {
            const bool mine = !(taken >> p & 1) && lane + RL_WAVE * p < choices && choice[p] == best;
            const unsigned long long all = __ballot(mine);
            if (!found && all) {
                found = true;
                if (mine && __ffsll(all) - 1 == lane) taken |= 1u << p;
            }
        }
    }
    float* dst = out + (size_t)t * (experts + 2);
    float returned = 0.f;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
        const int e = lane + RL_WAVE * p;
        const float weight = (taken >> p & 1) ? s[p] * scale : 0.f;
        if (e < experts)
            dst[e] = weight;
        else if (e < choices)
            returned += weight;
    }
    returned = sum_over_wave(returned);
    if (lane == 0) {
        dst[experts] = gate ? 1.f / (1.f + expf(-z[choices])) : 1.f;
        dst[experts + 1] = returned;
    }
}

template <typename T, typename W>
static int launch(const T* x, const W* w, const float* correction, float* out, int tokens, int k, int experts,
                  int identity, int gate, int top, float scale, hipStream_t stream) {
    const int choices = experts + identity;
    const int row_blocks = (choices + gate + 15) / 16;
    const size_t lds = sizeof(float) * TOKENS * ((row_blocks + BLOCKS - 1) / BLOCKS * BLOCKS * 16 + 1);
    dim3 grid((tokens + TOKENS - 1) / TOKENS), block(WAVES * RL_WAVE);
#define RL_CHOOSE(WHOLE, PER)                                                                                        \
    do {                                                                                                             \
        auto kernel = choose_experts_kernel<T, W, WHOLE, PER>;                                                       \
        /* (beyond 64 KB of LDS together with the kernel's own a launch has to ask) */                               \
        if (lds > 24 * 1024 &&                                                                                       \
            hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return RL_ERR_LAUNCH;                                                                                    \
        hipLaunchKernelGGL(kernel, grid, block, lds, stream, x, w, correction, out, tokens, k, experts, identity, gate, \
                           top, scale);                                                                              \
    } while (0)
#define RL_CHOOSE_PER(WHOLE)             \
    do {                                 \
        if (choices <= RL_WAVE)          \
            RL_CHOOSE(WHOLE, 1);         \
        else if (choices <= 4 * RL_WAVE) \
            RL_CHOOSE(WHOLE, 4);         \
        else                             \
            RL_CHOOSE(WHOLE, 16);        \
    } while (0)
    if (k % (sizeof(W) == 2 ? 32 : 16) == 0)
        RL_CHOOSE_PER(true);
    else
        RL_CHOOSE_PER(false);
#undef RL_CHOOSE_PER
#undef RL_CHOOSE
    return rl_launch_status();
}

}  // namespace router

// w: [experts + identity + gate, k], float32, or bfloat16 where x is; correction: [experts + identity] or null;
// out: [tokens, experts + 2]
extern "C" int rl_choose_experts(const void* x, const void* w, const float* correction, float* out, int tokens, int k,
                                 int experts, int identity, int gate, int top, float scale, int act_type, int w_type,
                                 hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (k < 1 || experts < 1 || identity < 0 || (gate != 0 && gate != 1) || experts + identity > router::MAX_CHOICES ||
        top < 1 || top > experts + identity)
        return RL_ERR_ARG;
    if (act_type == RL_F32 && w_type == RL_F32)
        return router::launch((const float*)x, (const float*)w, correction, out, tokens, k, experts, identity, gate, top,
                              scale, stream);
    if (act_type == RL_BF16 && w_type == RL_F32)
        return router::launch((const bf16_t*)x, (const float*)w, correction, out, tokens, k, experts, identity, gate, top,
                              scale, stream);
    if (act_type == RL_BF16 && w_type == RL_BF16)
        return router::launch((const bf16_t*)x, (const bf16_t*)w, correction, out, tokens, k, experts, identity, gate, top,
                              scale, stream);
    return RL_ERR_ARG;
}
