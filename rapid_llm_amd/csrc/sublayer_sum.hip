// The norm behind a layer whose sub-layers read the same rows: what they return joins the stream and
// the stream's rows are normed, in one kernel, float32 throughout:
//   residual += factor * (sum of terms + c_t x_t)        out = residual * rsqrt(mean(residual^2) + eps) * weight
// A term is a row y (+ bias) of a product, as it is or (with a weight of its own) divided by its root
// mean square and multiplied by that weight; up to three.  x is a row (the sub-layers' input) and c_t
// one number a token.  `rows` (optional) selects which rows are normed, packed in order; the stream
// is then not written back (whoever selects rows is the last to read it).
#include "common.h"

namespace sublayer_sum {

constexpr int TERMS = 3;

template <typename T>
struct Terms {
    const T* y[TERMS];           // null: no such term
    const float* bias[TERMS];    // null: none
    const float* weight[TERMS];  // null: the term is added as it is
    const T* x;                  // null: no such row
    const float* c;              // token t's number is c[t * c_stride]
    int c_stride;
    float eps, factor;
};

template <typename T>
struct alignas(sizeof(T) * 4) Quad {
    T v[4];
};

// sums over the workgroup of N values at once (scratch: [N][16])
template <int N>
__device__ inline void block_sums(float (&v)[N], float (*scratch)[16]) {
    const int lane = threadIdx.x & (RL_WAVE - 1), wave = threadIdx.x / RL_WAVE;
    const int waves = (blockDim.x + RL_WAVE - 1) / RL_WAVE;
#pragma unroll
    for (int n = 0; n < N; ++n) {
        v[n] = wave_sum(v[n]);
        if (lane == 0) scratch[n][wave] = v[n];
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < N; ++n) {
        float total = 0.f;
        for (int i = 0; i < waves; ++i) total += scratch[n][i];
        v[n] = total;
    }
}

// four channels a thread and access; a row of up to 4 * CHUNKS * blockDim elements stays in registers
template <typename T, int CHUNKS>
__global__ __launch_bounds__(1024) void sum_norm_vec_kernel(float* __restrict__ residual, Terms<T> in,
                                                            const float* __restrict__ weight, T* __restrict__ out,
                                                            const int* __restrict__ rows, int hidden, float eps) {
    __shared__ float scratch[TERMS][16], scratch1[1][16];
    const int r = blockIdx.x, row = rows ? rows[r] : r;
    const int nvec = hidden >> 2;
    float4* res = reinterpret_cast<float4*>(residual + (size_t)row * hidden);
    float4 val[CHUNKS], sum[CHUNKS], y[TERMS][CHUNKS];
    float ss[TERMS] = {0.f, 0.f, 0.f};
    const float c = in.x ? in.c[(size_t)row * in.c_stride] : 0.f;
#pragma unroll
    for (int k = 0; k < CHUNKS; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        if (i >= nvec) continue;
        val[k] = res[i];
        sum[k] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (in.x) {
            const Quad<T> q = reinterpret_cast<const Quad<T>*>(in.x + (size_t)row * hidden)[i];
            sum[k] = make_float4(c * to_float(q.v[0]), c * to_float(q.v[1]), c * to_float(q.v[2]), c * to_float(q.v[3]));
        }
#pragma unroll
        for (int t = 0; t < TERMS; ++t) {
            if (!in.y[t]) continue;
            const Quad<T> q = reinterpret_cast<const Quad<T>*>(in.y[t] + (size_t)row * hidden)[i];
            float4 v = make_float4(to_float(q.v[0]), to_float(q.v[1]), to_float(q.v[2]), to_float(q.v[3]));
            if (in.bias[t]) {
                const float4 b = reinterpret_cast<const float4*>(in.bias[t])[i];
                v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
            }
            y[t][k] = v;
            ss[t] += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    }
    if (in.weight[0] || in.weight[1] || in.weight[2]) block_sums<TERMS>(ss, scratch);
    float total[1] = {0.f};
    float rr[TERMS];
#pragma unroll
    for (int t = 0; t < TERMS; ++t) rr[t] = rsqrtf(ss[t] / (float)hidden + in.eps);
#pragma unroll
    for (int k = 0; k < CHUNKS; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        if (i >= nvec) continue;
#pragma unroll
        for (int t = 0; t < TERMS; ++t) {
            if (!in.y[t]) continue;
            const float4 v = y[t][k];
            if (in.weight[t]) {
                const float4 w = reinterpret_cast<const float4*>(in.weight[t])[i];
                sum[k].x += v.x * rr[t] * w.x; sum[k].y += v.y * rr[t] * w.y;
                sum[k].z += v.z * rr[t] * w.z; sum[k].w += v.w * rr[t] * w.w;
            } else {
                sum[k].x += v.x; sum[k].y += v.y; sum[k].z += v.z; sum[k].w += v.w;
            }
        }
        float4 v = val[k];
        v.x = fmaf(in.factor, sum[k].x, v.x); v.y = fmaf(in.factor, sum[k].y, v.y);
        v.z = fmaf(in.factor, sum[k].z, v.z); v.w = fmaf(in.factor, sum[k].w, v.w);
        if (!rows) res[i] = v;
        val[k] = v;
        total[0] += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
    }
    if (!out) return;  // (the same for every thread)
    block_sums<1>(total, scratch1);
    const float rrms = rsqrtf(total[0] / (float)hidden + eps);
#pragma unroll
    for (int k = 0; k < CHUNKS; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        if (i >= nvec) continue;
        const float4 w = reinterpret_cast<const float4*>(weight)[i];
        Quad<T> o;
        o.v[0] = from_float<T>(val[k].x * rrms * w.x);
        o.v[1] = from_float<T>(val[k].y * rrms * w.y);
        o.v[2] = from_float<T>(val[k].z * rrms * w.z);
        o.v[3] = from_float<T>(val[k].w * rrms * w.w);
        reinterpret_cast<Quad<T>*>(out + (size_t)r * hidden)[i] = o;
    }
}

// any width: three passes over the row
template <typename T>
__global__ __launch_bounds__(512) void sum_norm_kernel(float* __restrict__ residual, Terms<T> in,
                                                       const float* __restrict__ weight, T* __restrict__ out,
                                                       const int* __restrict__ rows, int hidden, float eps) {
    __shared__ float scratch[TERMS][16], scratch1[1][16];
    const int r = blockIdx.x, row = rows ? rows[r] : r;
    float* res = residual + (size_t)row * hidden;
    auto term = [&](int t, int i) -> float {
        const float v = to_float(in.y[t][(size_t)row * hidden + i]);
        return in.bias[t] ? v + in.bias[t][i] : v;
    };
    float ss[TERMS] = {0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < TERMS; ++t)
        if (in.y[t] && in.weight[t])
            for (int i = threadIdx.x; i < hidden; i += blockDim.x) ss[t] += term(t, i) * term(t, i);
    block_sums<TERMS>(ss, scratch);
    float rr[TERMS];
#pragma unroll
    for (int t = 0; t < TERMS; ++t) rr[t] = rsqrtf(ss[t] / (float)hidden + in.eps);
    const float c = in.x ? in.c[(size_t)row * in.c_stride] : 0.f;
    auto value = [&](int i) -> float {
        float sum = in.x ? c * to_float(in.x[(size_t)row * hidden + i]) : 0.f;
#pragma unroll
        for (int t = 0; t < TERMS; ++t)
            if (in.y[t]) sum += in.weight[t] ? term(t, i) * rr[t] * in.weight[t][i] : term(t, i);
        return fmaf(in.factor, sum, res[i]);
    };
    float total[1] = {0.f};
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float v = value(i);
        total[0] += v * v;
    }
    block_sums<1>(total, scratch1);
    const float rrms = rsqrtf(total[0] / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float v = value(i);
        if (!rows) res[i] = v;
        if (out) out[(size_t)r * hidden + i] = from_float<T>(v * rrms * weight[i]);
    }
}

template <typename T>
static int launch(float* residual, const Terms<T>& in, const float* weight, T* out, const int* rows, int out_rows,
                  int hidden, float eps, hipStream_t stream) {
    dim3 grid(out_rows);
    if (hidden % 4 == 0 && hidden <= 16 * 1024) {
        const int threads = (hidden / 4 + RL_WAVE - 1) / RL_WAVE * RL_WAVE;
        if (threads <= 1024)
            hipLaunchKernelGGL((sum_norm_vec_kernel<T, 1>), grid, dim3(threads), 0, stream, residual, in, weight, out, rows,
                               hidden, eps);
        else
            hipLaunchKernelGGL((sum_norm_vec_kernel<T, 4>), grid, dim3(1024), 0, stream, residual, in, weight, out, rows,
                               hidden, eps);
    } else {
        hipLaunchKernelGGL(sum_norm_kernel<T>, grid, dim3(hidden >= 2048 ? 512 : 256), 0, stream, residual, in, weight, out,
                           rows, hidden, eps);
    }
    return rl_launch_status();
}

template <typename T>
static int run(float* residual, const void* const* y, const float* const* bias, const float* const* term_weight,
               const void* x, const float* c, int c_stride, float term_eps, float factor, const float* weight, void* out,
               const int* rows, int out_rows, int hidden, float eps, hipStream_t stream) {
    Terms<T> in;
    for (int t = 0; t < TERMS; ++t) {
        in.y[t] = (const T*)y[t];
        in.bias[t] = y[t] ? bias[t] : nullptr;
        in.weight[t] = y[t] ? term_weight[t] : nullptr;
    }
    in.x = (const T*)x;
    in.c = c;
    in.c_stride = c_stride;
    in.eps = term_eps;
    in.factor = factor;
    return launch<T>(residual, in, weight, (T*)out, rows, out_rows, hidden, eps, stream);
}

}  // namespace sublayer_sum

extern "C" int rl_sublayer_sum_norm(float* residual, const void* y0, const float* b0, const float* w0, const void* y1,
                                    const float* b1, const float* w1, const void* y2, const float* b2, const float* w2,
                                    const void* x, const float* c, int c_stride, float term_eps, float factor,
                                    const float* weight, void* out, const int* rows, int out_rows, int hidden, float eps,
                                    int act_type, hipStream_t stream) {
    if (out_rows <= 0) return RL_OK;
    if (hidden < 1 || (x && (!c || c_stride < 1)) || (out && !weight) || (!out && rows)) return RL_ERR_ARG;
    const void* y[] = {y0, y1, y2};
    const float* bias[] = {b0, b1, b2};
    const float* term_weight[] = {w0, w1, w2};
    if (act_type == RL_F32)
        return sublayer_sum::run<float>(residual, y, bias, term_weight, x, c, c_stride, term_eps, factor, weight, out, rows,
                                        out_rows, hidden, eps, stream);
    if (act_type == RL_BF16)
        return sublayer_sum::run<bf16_t>(residual, y, bias, term_weight, x, c, c_stride, term_eps, factor, weight, out,
                                         rows, out_rows, hidden, eps, stream);
    return RL_ERR_ARG;
}
