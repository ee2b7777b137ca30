// Router of a mixture whose experts are chosen by corrected scores, with experts that return their
// input and a gate for a shared expert, in one kernel, float32 throughout:
//   z = W x over `experts` experts with tensors, `identity` experts without, and, with `gate`, one more row;
//   s = softmax(z) over the experts + identity; chosen: the `top` largest s + correction (the lower
//   index wins a tie); a chosen expert's weight is s * scale (not divided by anything).
// A token's row of `out` has experts + 2 entries: the experts' weights (0 for those not chosen), the
// sigmoid of the gate's row (1 without one), and the sum of the chosen identity experts' weights.
//
// A workgroup takes 16 tokens.  The product runs on the true 32-bit matrix instruction
// (v_mfma_f32_16x16x4_f32), its inner dimension dealt to 16 waves in steps of 16; their shares are
// added in the order of the waves, so a token's logits do not depend on what else is in the step.
// Then every wave takes a token and chooses.
#include "common.h"

namespace router {

constexpr int TOKENS = 16;
constexpr int WAVES = 16;
constexpr int BLOCKS = 2;  // of 16 rows of W, multiplied with what is read of x
constexpr int MAX_CHOICES = 1024;
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <typename T>
struct alignas(sizeof(T) * 4) Quad {
    T v[4];
};

// elements i .. i + 3 of a row of k; WHOLE: they are all there (k is a multiple of 16)
template <bool WHOLE, typename T>
__device__ inline Quad<T> quad_at(const T* __restrict__ row, int i, int k) {
    if constexpr (WHOLE) return *reinterpret_cast<const Quad<T>*>(row + i);
    Quad<T> q;
#pragma unroll
    for (int e = 0; e < 4; ++e) q.v[e] = i + e < k ? row[i + e] : from_float<T>(0.f);
    return q;
}

template <typename T, bool WHOLE, int PER>
__global__ __launch_bounds__(WAVES* RL_WAVE) void choose_experts_kernel(
    const T* __restrict__ x, const float* __restrict__ w, const float* __restrict__ correction, float* __restrict__ out,
    int tokens, int k, int experts, int identity, int gate, int top, float scale) {
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
        const float* wr[BLOCKS];
#pragma unroll
        for (int b = 0; b < BLOCKS; ++b) {
            acc[b] = (f32x4){0.f, 0.f, 0.f, 0.f};
            wr[b] = w + (size_t)min(16 * (b0 + b) + r16, rows - 1) * k;  // (beyond the rows: a real one, not used)
        }
        // four steps' operands are asked for together (a step of a few tokens is all latency here)
        for (int i0 = 16 * wave; i0 < k; i0 += 4 * 16 * WAVES) {
            Quad<T> xq[4];
            Quad<float> wq[4][BLOCKS];
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int i = i0 + q * 16 * WAVES;
                const int at = (i < k ? i : i0) + 4 * g;  // (beyond the row: the first step's again, not used)
                xq[q] = quad_at<WHOLE>(xr, at, k);
#pragma unroll
                for (int b = 0; b < BLOCKS; ++b) wq[q][b] = quad_at<WHOLE>(wr[b], at, k);
            }
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                if (i0 + q * 16 * WAVES >= k) continue;
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int b = 0; b < BLOCKS; ++b)
                        acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(to_float(xq[q].v[e]), wq[q][b].v[e], acc[b], 0, 0, 0);
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
    m = wave_max(m);
    float total = 0.f;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
        s[p] = expf(s[p] - m);
        total += s[p];
    }
    total = wave_sum(total);
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
        int at = 0x7fffffff;
#pragma unroll
        for (int p = 0; p < PER; ++p)
            if (!(taken >> p & 1) && choice[p] > best) {
                best = choice[p];
                at = lane + RL_WAVE * p;
            }
#pragma unroll
        for (int o = RL_WAVE / 2; o > 0; o >>= 1) {
            const float other = __shfl_xor(best, o, RL_WAVE);
            const int other_at = __shfl_xor(at, o, RL_WAVE);
            if (other > best || (other == best && other_at < at)) {
                best = other;
                at = other_at;
            }
        }
        if (at != 0x7fffffff && (at & (RL_WAVE - 1)) == lane) taken |= 1u << (at / RL_WAVE);
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
    returned = wave_sum(returned);
    if (lane == 0) {
        dst[experts] = gate ? 1.f / (1.f + expf(-z[choices])) : 1.f;
        dst[experts + 1] = returned;
    }
}

template <typename T>
static int launch(const T* x, const float* w, const float* correction, float* out, int tokens, int k, int experts,
                  int identity, int gate, int top, float scale, hipStream_t stream) {
    const int choices = experts + identity;
    const int row_blocks = (choices + gate + 15) / 16;
    const size_t lds = sizeof(float) * TOKENS * ((row_blocks + BLOCKS - 1) / BLOCKS * BLOCKS * 16 + 1);
    dim3 grid((tokens + TOKENS - 1) / TOKENS), block(WAVES * RL_WAVE);
#define RL_CHOOSE(WHOLE, PER)                                                                                        \
    do {                                                                                                             \
        auto kernel = choose_experts_kernel<T, WHOLE, PER>;                                                          \
        /* (beyond 64 KB of LDS together with the kernel's own a launch has to ask) */                               \
        if (lds > 24 * 1024 &&                                                                                       \
            hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
            return RL_ERR_LAUNCH;                                                                                    \
        hipLaunchKernelGGL(kernel, grid, block, lds, stream, x, w, correction, out, tokens, k, experts, identity, gate, \
                           top, scale);                                                                              \
    } while (0)
#define RL_CHOOSE_PER(WHOLE)         \
    do {                             \
        if (choices <= RL_WAVE)      \
            RL_CHOOSE(WHOLE, 1);     \
        else if (choices <= 4 * RL_WAVE) \
            RL_CHOOSE(WHOLE, 4);     \
        else                         \
            RL_CHOOSE(WHOLE, 16);    \
    } while (0)
    if (k % 16 == 0)
        RL_CHOOSE_PER(true);
    else
        RL_CHOOSE_PER(false);
#undef RL_CHOOSE_PER
#undef RL_CHOOSE
    return rl_launch_status();
}

}  // namespace router

// w: [experts + identity + gate, k]; correction: [experts + identity] or null; out: [tokens, experts + 2]
extern "C" int rl_choose_experts(const void* x, const float* w, const float* correction, float* out, int tokens, int k,
                                 int experts, int identity, int gate, int top, float scale, int act_type,
                                 hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (k < 1 || experts < 1 || identity < 0 || (gate != 0 && gate != 1) || experts + identity > router::MAX_CHOICES ||
        top < 1 || top > experts + identity)
        return RL_ERR_ARG;
    if (act_type == RL_F32)
        return router::launch<float>((const float*)x, w, correction, out, tokens, k, experts, identity, gate, top, scale,
                                     stream);
    if (act_type == RL_BF16)
        return router::launch<bf16_t>((const bf16_t*)x, w, correction, out, tokens, k, experts, identity, gate, top,
                                      scale, stream);
    return RL_ERR_ARG;
}
