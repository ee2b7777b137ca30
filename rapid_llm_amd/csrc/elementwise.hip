// Row-wise kernels of the decoder: embedding gather, residual-add + RMSNorm, SwiGLU,
// rotation tables, the fused per-head norm + rotation + cache write, and a type cast.
// All arithmetic is float32; the element type only decides loads and stores.
#include "common.h"

// --------------------------------------------------------------------------- //
// embedding: residual[t, :] = table[ids[t], :] * scale   (float32 residual stream)
// rapid_llm/modules/vocab_parallel.py:102-103
// With `inv_freq` (hidden / 2 float32 frequencies) a sinusoidal position vector is added:
// channel 2i gets sin(a), channel 2i + 1 cos(a), a = positions[t] * inv_freq[i] as a float32
// product; sine and cosine of that angle are evaluated in double.
// With `pos_table` (rows of the table's type, one a position) row positions[t] is added, unscaled.
// --------------------------------------------------------------------------- //
__device__ inline float sinusoid_channel(int pos, int channel, const float* __restrict__ inv_freq) {
    const float angle = (float)pos * inv_freq[channel >> 1];
    return (float)((channel & 1) ? cos((double)angle) : sin((double)angle));
}

// A negative id -(r + 1) stands for "the token chosen in row r of the previous step", which
// the host may not have seen yet: it is read from `fed` (the sampling kernels' output)
// (rapid_llm/engine/scheduler.py:241-249: the placeholder a device-side gather replaces).
template <typename W>
__global__ void embed_kernel(const int* __restrict__ ids, const int* __restrict__ fed, int fed_rows,
                             const W* __restrict__ table, float* __restrict__ out, int hidden,
                             int vocab, float scale, const int* __restrict__ positions,
                             const float* __restrict__ inv_freq, const W* __restrict__ pos_table, int pos_rows) {
    const int t = blockIdx.x;
    const int pos = (inv_freq || pos_table) ? positions[t] : 0;
    // positions are validated on the host; one beyond the table reads its last row rather than faulting
    const W* prow = pos_table ? pos_table + (size_t)min(max(pos, 0), pos_rows - 1) * hidden : nullptr;
    int id = ids[t];
    if (id < 0 && fed && -id - 1 < fed_rows) id = fed[-id - 1];
    // ids are validated on the host; an id outside the table reads row 0 rather than faulting
    if (id < 0 || id >= vocab) id = 0;
    const W* row = table + (size_t)id * hidden;
    float* dst = out + (size_t)t * hidden;
    constexpr int VEC = 16 / sizeof(W);  // elements of one 16-byte read
    if (hidden % VEC == 0) {
        struct alignas(16) Pack {
            W v[VEC];
        };
        for (int i = threadIdx.x * VEC; i < hidden; i += blockDim.x * VEC) {
            const Pack p = *reinterpret_cast<const Pack*>(row + i);
            Pack pp;
            if (prow) pp = *reinterpret_cast<const Pack*>(prow + i);
#pragma unroll
            for (int j = 0; j < VEC; j += 4) {
                float4 v = make_float4(to_float(p.v[j]) * scale, to_float(p.v[j + 1]) * scale,
                                       to_float(p.v[j + 2]) * scale, to_float(p.v[j + 3]) * scale);
                if (prow) {
                    v.x += to_float(pp.v[j]);
                    v.y += to_float(pp.v[j + 1]);
                    v.z += to_float(pp.v[j + 2]);
                    v.w += to_float(pp.v[j + 3]);
                }
                if (inv_freq) {
                    v.x += sinusoid_channel(pos, i + j, inv_freq);
                    v.y += sinusoid_channel(pos, i + j + 1, inv_freq);
                    v.z += sinusoid_channel(pos, i + j + 2, inv_freq);
                    v.w += sinusoid_channel(pos, i + j + 3, inv_freq);
                }
                *reinterpret_cast<float4*>(dst + i + j) = v;
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float v = to_float(row[i]) * scale;
        if (prow) v += to_float(prow[i]);
        if (inv_freq) v += sinusoid_channel(pos, i, inv_freq);
        dst[i] = v;
    }
}

extern "C" int rl_embed(const int* ids, const int* fed, int fed_rows, const void* table,
                        int table_type, float* out, int tokens, int hidden, int vocab, float scale,
                        const int* positions, const float* inv_freq, const void* pos_table, int pos_rows,
                        hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if ((inv_freq || pos_table) && !positions) return RL_ERR_ARG;
    if (pos_table && pos_rows < 1) return RL_ERR_ARG;
    dim3 grid(tokens), block(256);
    if (table_type == RL_F32)
        hipLaunchKernelGGL(embed_kernel<float>, grid, block, 0, stream, ids, fed, fed_rows,
                           (const float*)table, out, hidden, vocab, scale, positions, inv_freq,
                           (const float*)pos_table, pos_rows);
    else if (table_type == RL_BF16)
        hipLaunchKernelGGL(embed_kernel<bf16_t>, grid, block, 0, stream, ids, fed, fed_rows,
                           (const bf16_t*)table, out, hidden, vocab, scale, positions, inv_freq,
                           (const bf16_t*)pos_table, pos_rows);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// residual += delta (+ bias, float32 [hidden]: that of the product that delta is, or null), float32,
// in place; out = residual * rsqrt(mean(residual^2)+eps) * w
// One block per produced row; `rows` (optional) selects which residual rows are produced,
// packed in order.  rapid_llm/kernels/ops/layernorm/skip_rmsnorm.py:51-85: the sum is
// formed in float32 and the norm reads the unrounded sum.
// --------------------------------------------------------------------------- //
template <typename T>
__global__ void add_rmsnorm_kernel(float* __restrict__ residual, const T* __restrict__ delta,
                                   const float* __restrict__ weight, T* __restrict__ out,
                                   const int* __restrict__ rows, int hidden, float eps,
                                       const float* __restrict__ bias) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int row = rows ? rows[r] : r;
    float* res = residual + (size_t)row * hidden;
    const T* dl = delta ? delta + (size_t)row * hidden : nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float v = res[i];
        if (dl) {
            v += to_float(dl[i]);
            if (bias) v += bias[i];
            res[i] = v;
        }
        ss += v * v;
    }
    ss = block_sum(ss, scratch);
    const float rrms = rsqrtf(ss / (float)hidden + eps);
    T* o = out + (size_t)r * hidden;
    // each thread re-reads exactly the elements it wrote above
    for (int i = threadIdx.x; i < hidden; i += blockDim.x)
        o[i] = from_float<T>(res[i] * rrms * weight[i]);
}

// The same with four elements per thread and load: a row of up to 16 * blockDim elements
// stays in registers between the two passes, so a row costs one round trip to memory.  With
// few rows (decode) the kernel's time is that latency, not bandwidth.
template <typename T>
struct alignas(sizeof(T) * 4) Vec4 {
    T v[4];
};

template <typename T, int CHUNKS>
__global__ void add_rmsnorm_vec_kernel(float* __restrict__ residual, const T* __restrict__ delta,
                                       const float* __restrict__ weight, T* __restrict__ out,
                                       const int* __restrict__ rows, int hidden, float eps,
                                       const float* __restrict__ bias) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int row = rows ? rows[r] : r;
    float4* res = reinterpret_cast<float4*>(residual + (size_t)row * hidden);
    const Vec4<T>* dl = delta ? reinterpret_cast<const Vec4<T>*>(delta + (size_t)row * hidden) : nullptr;
    const int nvec = hidden >> 2;
    const float4* w4 = reinterpret_cast<const float4*>(weight);
    float4 val[CHUNKS], wt[CHUNKS];
    float ss = 0.f;
    // the weights are read before the sum, not after its barrier: one wait less in a kernel
    // that is all latency when it has a handful of rows
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) wt[c] = w4[i];
    }
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            float4 v = res[i];
            if (dl) {
                const Vec4<T> d = dl[i];
                v.x += to_float(d.v[0]);
                v.y += to_float(d.v[1]);
                v.z += to_float(d.v[2]);
                v.w += to_float(d.v[3]);
                if (bias) {
                    const float4 b = reinterpret_cast<const float4*>(bias)[i];
                    v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
                }
                res[i] = v;
            }
            val[c] = v;
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    }
    ss = block_sum(ss, scratch);
    const float rrms = rsqrtf(ss / (float)hidden + eps);
    Vec4<T>* o = reinterpret_cast<Vec4<T>*>(out + (size_t)r * hidden);
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            const float4 w = wt[c];
            Vec4<T> y;
            y.v[0] = from_float<T>(val[c].x * rrms * w.x);
            y.v[1] = from_float<T>(val[c].y * rrms * w.y);
            y.v[2] = from_float<T>(val[c].z * rrms * w.z);
            y.v[3] = from_float<T>(val[c].w * rrms * w.w);
            o[i] = y;
        }
    }
}

template <typename T>
static void launch_add_rmsnorm(float* residual, const T* delta, const float* weight, T* out,
                               const int* rows, int out_rows, int hidden, float eps,
                               const float* bias, hipStream_t stream) {
    dim3 grid(out_rows);
    if (hidden % 4 == 0 && hidden <= 16 * 1024) {
        const int nvec = hidden / 4;
        // one chunk per thread while the block stays within 1024 threads, then up to four
        int threads = ((nvec + RL_WAVE - 1) / RL_WAVE) * RL_WAVE;
        if (threads <= 1024) {
            hipLaunchKernelGGL((add_rmsnorm_vec_kernel<T, 1>), grid, dim3(threads), 0, stream,
                               residual, delta, weight, out, rows, hidden, eps, bias);
        } else {
            hipLaunchKernelGGL((add_rmsnorm_vec_kernel<T, 4>), grid, dim3(1024), 0, stream,
                               residual, delta, weight, out, rows, hidden, eps, bias);
        }
        return;
    }
    int threads = hidden >= 2048 ? 512 : (hidden >= 512 ? 256 : 64);
    hipLaunchKernelGGL(add_rmsnorm_kernel<T>, grid, dim3(threads), 0, stream, residual, delta,
                       weight, out, rows, hidden, eps, bias);
}

extern "C" int rl_add_rmsnorm(float* residual, const void* delta, const float* weight, void* out,
                              const int* rows, int out_rows, int hidden, float eps, int act_type,
                              const float* bias, hipStream_t stream) {
    if (out_rows <= 0) return RL_OK;
    if (act_type == RL_F32)
        launch_add_rmsnorm<float>(residual, (const float*)delta, weight, (float*)out, rows,
                                  out_rows, hidden, eps, bias, stream);
    else if (act_type == RL_BF16)
        launch_add_rmsnorm<bf16_t>(residual, (const bf16_t*)delta, weight, (bf16_t*)out, rows,
                                   out_rows, hidden, eps, bias, stream);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// A sub-layer whose output passes a norm of its own before it joins the stream:
//   residual += y * rsqrt(mean(y^2) + eps_y) * w_y        (float32, in place)
//   out       = residual * rsqrt(mean(residual^2) + eps) * w   (skipped when out is null)
// One block per produced row, `rows` as in rl_add_rmsnorm.  Both statistics and the sum are
// float32; y is read once and stays in registers between its two passes (rows of up to
// 8 * blockDim elements, else it is read again).
// --------------------------------------------------------------------------- //
template <typename T, int PER>
__global__ void normed_add_rmsnorm_kernel(float* __restrict__ residual, const T* __restrict__ y,
                                          const float* __restrict__ w_y, float eps_y,
                                          const float* __restrict__ weight, T* __restrict__ out,
                                          const int* __restrict__ rows, int hidden, float eps) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int row = rows ? rows[r] : r;
    float* res = residual + (size_t)row * hidden;
    const T* yr = y + (size_t)row * hidden;
    float val[PER];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < PER; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        val[c] = i < hidden ? to_float(yr[i]) : 0.f;
        ss += val[c] * val[c];
    }
    for (int i = threadIdx.x + PER * blockDim.x; i < hidden; i += blockDim.x) {
        const float v = to_float(yr[i]);
        ss += v * v;
    }
    ss = block_sum(ss, scratch);
    const float rr_y = rsqrtf(ss / (float)hidden + eps_y);
    float s2 = 0.f;
#pragma unroll
    for (int c = 0; c < PER; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < hidden) {
            val[c] = res[i] + val[c] * rr_y * w_y[i];
            res[i] = val[c];
            s2 += val[c] * val[c];
        }
    }
    for (int i = threadIdx.x + PER * blockDim.x; i < hidden; i += blockDim.x) {
        const float v = res[i] + to_float(yr[i]) * rr_y * w_y[i];
        res[i] = v;
        s2 += v * v;
    }
    if (!out) return;
    s2 = block_sum(s2, scratch);
    const float rrms = rsqrtf(s2 / (float)hidden + eps);
    T* o = out + (size_t)r * hidden;
#pragma unroll
    for (int c = 0; c < PER; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < hidden) o[i] = from_float<T>(val[c] * rrms * weight[i]);
    }
    // each thread re-reads exactly the elements it wrote above
    for (int i = threadIdx.x + PER * blockDim.x; i < hidden; i += blockDim.x)
        o[i] = from_float<T>(res[i] * rrms * weight[i]);
}

// The same with four elements a thread and load, a row of up to 16 * blockDim elements held in
// registers from its first read to its last use.
template <typename T, int CHUNKS>
__global__ void normed_add_rmsnorm_vec_kernel(float* __restrict__ residual, const T* __restrict__ y,
                                              const float* __restrict__ w_y, float eps_y,
                                              const float* __restrict__ weight, T* __restrict__ out,
                                              const int* __restrict__ rows, int hidden, float eps) {
    __shared__ float scratch[16];
    const int r = blockIdx.x;
    const int row = rows ? rows[r] : r;
    float4* res = reinterpret_cast<float4*>(residual + (size_t)row * hidden);
    const Vec4<T>* yr = reinterpret_cast<const Vec4<T>*>(y + (size_t)row * hidden);
    const float4* wy4 = reinterpret_cast<const float4*>(w_y);
    const float4* w4 = reinterpret_cast<const float4*>(weight);
    const int nvec = hidden >> 2;
    float4 val[CHUNKS], old[CHUNKS], wy[CHUNKS], wt[CHUNKS];
    float ss = 0.f;
    // everything the row needs is asked for before the first sum's barrier
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            const Vec4<T> v = yr[i];
            val[c] = make_float4(to_float(v.v[0]), to_float(v.v[1]), to_float(v.v[2]), to_float(v.v[3]));
            old[c] = res[i];
            wy[c] = wy4[i];
            if (out) wt[c] = w4[i];
            ss += val[c].x * val[c].x + val[c].y * val[c].y + val[c].z * val[c].z + val[c].w * val[c].w;
        }
    }
    ss = block_sum(ss, scratch);
    const float rr_y = rsqrtf(ss / (float)hidden + eps_y);
    float s2 = 0.f;
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            float4 v;
            v.x = old[c].x + val[c].x * rr_y * wy[c].x;
            v.y = old[c].y + val[c].y * rr_y * wy[c].y;
            v.z = old[c].z + val[c].z * rr_y * wy[c].z;
            v.w = old[c].w + val[c].w * rr_y * wy[c].w;
            res[i] = v;
            val[c] = v;
            s2 += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    }
    if (!out) return;
    s2 = block_sum(s2, scratch);
    const float rrms = rsqrtf(s2 / (float)hidden + eps);
    Vec4<T>* o = reinterpret_cast<Vec4<T>*>(out + (size_t)r * hidden);
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            Vec4<T> v;
            v.v[0] = from_float<T>(val[c].x * rrms * wt[c].x);
            v.v[1] = from_float<T>(val[c].y * rrms * wt[c].y);
            v.v[2] = from_float<T>(val[c].z * rrms * wt[c].z);
            v.v[3] = from_float<T>(val[c].w * rrms * wt[c].w);
            o[i] = v;
        }
    }
}

template <typename T>
static void launch_normed_add_rmsnorm(float* residual, const T* y, const float* w_y, float eps_y,
                                      const float* weight, T* out, const int* rows, int out_rows, int hidden,
                                      float eps, hipStream_t stream) {
    dim3 grid(out_rows);
    if (hidden % 4 == 0 && hidden <= 16 * 1024) {
        const int nvec = hidden / 4;
        const int threads = ((nvec + RL_WAVE - 1) / RL_WAVE) * RL_WAVE;
        if (threads <= 1024)
            hipLaunchKernelGGL((normed_add_rmsnorm_vec_kernel<T, 1>), grid, dim3(threads), 0, stream, residual, y,
                               w_y, eps_y, weight, out, rows, hidden, eps);
        else
            hipLaunchKernelGGL((normed_add_rmsnorm_vec_kernel<T, 4>), grid, dim3(1024), 0, stream, residual, y,
                               w_y, eps_y, weight, out, rows, hidden, eps);
        return;
    }
    const int threads = hidden >= 4096 ? 1024 : (hidden >= 1024 ? 512 : (hidden >= 256 ? 256 : 64));
    hipLaunchKernelGGL((normed_add_rmsnorm_kernel<T, 8>), grid, dim3(threads), 0, stream, residual, y, w_y, eps_y,
                       weight, out, rows, hidden, eps);
}

extern "C" int rl_normed_add_rmsnorm(float* residual, const void* y, const float* w_y, float eps_y,
                                     const float* weight, void* out, const int* rows, int out_rows,
                                     int hidden, float eps, int act_type, hipStream_t stream) {
    if (out_rows <= 0) return RL_OK;
    if (out && !weight) return RL_ERR_ARG;
    if (act_type == RL_F32)
        launch_normed_add_rmsnorm<float>(residual, (const float*)y, w_y, eps_y, weight, (float*)out, rows, out_rows,
                                         hidden, eps, stream);
    else if (act_type == RL_BF16)
        launch_normed_add_rmsnorm<bf16_t>(residual, (const bf16_t*)y, w_y, eps_y, weight, (bf16_t*)out, rows,
                                          out_rows, hidden, eps, stream);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// out[t] = [a[t] | b[t]] in the compute type: two float32 streams of `hidden` channels side by
// side, the operand of a product over both.
template <typename T>
__global__ void pair_rows_kernel(const float* __restrict__ a, const float* __restrict__ b,
                                 T* __restrict__ out, size_t total, int hidden) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const size_t t = idx / (2 * (size_t)hidden);
        const int c = (int)(idx - t * 2 * (size_t)hidden);
        out[idx] = from_float<T>(c < hidden ? a[t * hidden + c] : b[t * hidden + c - hidden]);
    }
}

// four channels a thread (hidden a multiple of 4); `total` counts groups of four
template <typename T>
__global__ void pair_rows_vec_kernel(const float4* __restrict__ a, const float4* __restrict__ b,
                                     Vec4<T>* __restrict__ out, size_t total, int hidden4) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const size_t t = idx / (2 * (size_t)hidden4);
        const int c = (int)(idx - t * 2 * (size_t)hidden4);
        const float4 v = c < hidden4 ? a[t * hidden4 + c] : b[t * hidden4 + c - hidden4];
        Vec4<T> o;
        o.v[0] = from_float<T>(v.x);
        o.v[1] = from_float<T>(v.y);
        o.v[2] = from_float<T>(v.z);
        o.v[3] = from_float<T>(v.w);
        out[idx] = o;
    }
}

extern "C" int rl_pair_rows(const float* a, const float* b, void* out, int tokens, int hidden,
                            int act_type, hipStream_t stream) {
    if (tokens <= 0 || hidden <= 0) return RL_OK;
    if (act_type != RL_F32 && act_type != RL_BF16) return RL_ERR_ARG;
    const bool vec = hidden % 4 == 0;
    const size_t total = (size_t)tokens * 2 * hidden / (vec ? 4 : 1);
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    dim3 grid((unsigned)blocks), block(256);
    if (vec && act_type == RL_F32)
        hipLaunchKernelGGL(pair_rows_vec_kernel<float>, grid, block, 0, stream, (const float4*)a, (const float4*)b,
                           (Vec4<float>*)out, total, hidden / 4);
    else if (vec)
        hipLaunchKernelGGL(pair_rows_vec_kernel<bf16_t>, grid, block, 0, stream, (const float4*)a, (const float4*)b,
                           (Vec4<bf16_t>*)out, total, hidden / 4);
    else if (act_type == RL_F32)
        hipLaunchKernelGGL(pair_rows_kernel<float>, grid, block, 0, stream, a, b, (float*)out, total, hidden);
    else
        hipLaunchKernelGGL(pair_rows_kernel<bf16_t>, grid, block, 0, stream, a, b, (bf16_t*)out, total, hidden);
    return rl_launch_status();
}

// The same norm where the delta arrives as `nparts` float32 runs of a product's K
// (parts[run][row][hidden], see rl_gemm_mid_parts): the runs are added in order, the sum is
// rounded to the activation type as a stored product would be, then added to the residual (with
// the product's bias, where it has one).
template <typename T, int CHUNKS>
__global__ void add_parts_rmsnorm_kernel(float* __restrict__ residual, const float* __restrict__ parts,
                                         int nparts, size_t part_stride,
                                         const float* __restrict__ weight, T* __restrict__ out,
                                         int hidden, float eps, const float* __restrict__ bias) {
    __shared__ float scratch[16];
    const int row = blockIdx.x;
    float4* res = reinterpret_cast<float4*>(residual + (size_t)row * hidden);
    const int nvec = hidden >> 2;
    const float4* w4 = reinterpret_cast<const float4*>(weight);
    float4 val[CHUNKS], wt[CHUNKS];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) wt[c] = w4[i];
    }
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            const float4* pr = reinterpret_cast<const float4*>(parts + (size_t)row * hidden) + i;
            float4 d = *pr;
            for (int r = 1; r < nparts; ++r) {
                const float4 e = *reinterpret_cast<const float4*>(
                    reinterpret_cast<const float*>(pr) + (size_t)r * part_stride);
                d.x += e.x;
                d.y += e.y;
                d.z += e.z;
                d.w += e.w;
            }
            float4 v = res[i];
            v.x += to_float(from_float<T>(d.x));
            v.y += to_float(from_float<T>(d.y));
            v.z += to_float(from_float<T>(d.z));
            v.w += to_float(from_float<T>(d.w));
            if (bias) {
                const float4 b = reinterpret_cast<const float4*>(bias)[i];
                v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
            }
            res[i] = v;
            val[c] = v;
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    }
    ss = block_sum(ss, scratch);
    const float rrms = rsqrtf(ss / (float)hidden + eps);
    Vec4<T>* o = reinterpret_cast<Vec4<T>*>(out + (size_t)row * hidden);
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int i = threadIdx.x + c * blockDim.x;
        if (i < nvec) {
            const float4 w = wt[c];
            Vec4<T> y;
            y.v[0] = from_float<T>(val[c].x * rrms * w.x);
            y.v[1] = from_float<T>(val[c].y * rrms * w.y);
            y.v[2] = from_float<T>(val[c].z * rrms * w.z);
            y.v[3] = from_float<T>(val[c].w * rrms * w.w);
            o[i] = y;
        }
    }
}

// parts [nparts, rows, hidden] float32, contiguous; bfloat16 rows out; hidden a multiple of 4 up to 16 K
extern "C" int rl_add_rmsnorm_parts(float* residual, const float* parts, int nparts,
                                    const float* weight, void* out, int rows, int hidden, float eps,
                                    const float* bias, hipStream_t stream) {
    if (rows <= 0) return RL_OK;
    if (nparts < 1 || hidden % 4 || hidden > 16 * 1024) return RL_ERR_ARG;
    const int nvec = hidden / 4;
    const int threads = ((nvec + RL_WAVE - 1) / RL_WAVE) * RL_WAVE;
    const size_t stride = (size_t)rows * hidden;
    if (threads <= 1024)
        hipLaunchKernelGGL((add_parts_rmsnorm_kernel<bf16_t, 1>), dim3(rows), dim3(threads), 0, stream,
                           residual, parts, nparts, stride, weight, (bf16_t*)out, hidden, eps, bias);
    else
        hipLaunchKernelGGL((add_parts_rmsnorm_kernel<bf16_t, 4>), dim3(rows), dim3(1024), 0, stream,
                           residual, parts, nparts, stride, weight, (bf16_t*)out, hidden, eps, bias);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// Gated activation on the packed [gate | up] row: out[:, j] = act(x[:, j], x[:, I + j]).
// limit <= 0: SwiGLU, silu(g) * u (rapid_llm/kernels/ops/activation/swiglu.py:91-121).
// limit > 0: the clamped variant, g' = min(g, limit), u' = clamp(u, -limit, limit),
// g' * sigmoid(alpha * g') * (u' + 1).  gelu: gelu(g) * u in gelu's tanh form.  `bias` (float32,
// [2 I]) is added to gate and up values as they are read.
// With `route` (float32 [tokens, experts]) the first experts * ff hidden units of a row are those
// of `experts` experts side by side, and expert e's are multiplied by route[t, e]; with
// `route_input` the gate and up values are multiplied by it instead, before the activation (an
// expert whose input was scaled: its two products are linear).
// --------------------------------------------------------------------------- //
template <typename T>
__global__ void swiglu_kernel(const T* __restrict__ gate_up, T* __restrict__ out, int inter,
                              size_t total, Glu glu, const float* __restrict__ route,
                              int experts, int ff, int route_input) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const size_t t = idx / inter;
        const int j = (int)(idx - t * inter);
        const T* row = gate_up + t * 2 * (size_t)inter;
        float g = to_float(row[j]);
        float u = to_float(row[inter + j]);
        if (glu.bias) {
            g += glu.bias[j];
            u += glu.bias[inter + j];
        }
        const float factor = (route && j < experts * ff) ? route[t * experts + j / ff] : 1.f;
        const float v = route_input ? glu_act(g * factor, u * factor, glu)
                                    : glu_act(g, u, glu) * factor;
        out[idx] = from_float<T>(v);
    }
}

// eight elements per thread (16-byte loads for bfloat16) when the width allows it
template <typename T>
struct alignas(sizeof(T) * 8) Vec8 {
    T v[8];
};

template <typename T>
__global__ void swiglu_vec_kernel(const T* __restrict__ gate_up, T* __restrict__ out, int inter,
                                  size_t total_vec, Glu glu, const float* __restrict__ route,
                                  int experts, int ff, int route_input) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    const int per_row = inter >> 3;
    for (; idx < total_vec; idx += step) {
        const size_t t = idx / per_row;
        const int j = (int)(idx - t * per_row) << 3;
        const T* row = gate_up + t * 2 * (size_t)inter;
        const Vec8<T> g = *reinterpret_cast<const Vec8<T>*>(row + j);
        const Vec8<T> u = *reinterpret_cast<const Vec8<T>*>(row + inter + j);
        // (with a route, an expert's hidden units are a multiple of 8: one factor a group)
        const float factor = (route && j < experts * ff) ? route[t * experts + j / ff] : 1.f;
        Vec8<float> gb = {}, ub = {};
        if (glu.bias) {
            gb = *reinterpret_cast<const Vec8<float>*>(glu.bias + j);
            ub = *reinterpret_cast<const Vec8<float>*>(glu.bias + inter + j);
        }
        Vec8<T> y;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float gi = to_float(g.v[i]) + gb.v[i], ui = to_float(u.v[i]) + ub.v[i];
            y.v[i] = from_float<T>(route_input ? glu_act(gi * factor, ui * factor, glu) : glu_act(gi, ui, glu) * factor);
        }
        *reinterpret_cast<Vec8<T>*>(out + t * (size_t)inter + j) = y;
    }
}

template <typename T>
static void launch_swiglu(const T* gate_up, T* out, int tokens, int inter, const Glu& glu,
                          const float* route, int experts, int ff, int route_input, hipStream_t stream) {
    if (inter % 8 == 0 && (!route || ff % 8 == 0)) {
        const size_t total = (size_t)tokens * (inter / 8);
        size_t blocks = (total + 255) / 256;
        if (blocks > 65536) blocks = 65536;
        hipLaunchKernelGGL(swiglu_vec_kernel<T>, dim3((unsigned)blocks), dim3(256), 0, stream,
                           gate_up, out, inter, total, glu, route, experts, ff, route_input);
        return;
    }
    const size_t total = (size_t)tokens * inter;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    hipLaunchKernelGGL(swiglu_kernel<T>, dim3((unsigned)blocks), dim3(256), 0, stream, gate_up, out,
                       inter, total, glu, route, experts, ff, route_input);
}

extern "C" int rl_swiglu(const void* gate_up, void* out, int tokens, int inter, int act_type,
                         float limit, float alpha, const float* route, int experts, int ff, int route_input,
                         int gelu, const float* bias, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (bias && route_input) return RL_ERR_ARG;  // a scaled input does not scale the bias
    const Glu glu = {limit, alpha, gelu, bias};
    if (route && (experts < 1 || ff < 1 || (long)experts * ff > inter)) return RL_ERR_ARG;
    if (route_input && !route) return RL_ERR_ARG;
    if (act_type == RL_F32)
        launch_swiglu<float>((const float*)gate_up, (float*)out, tokens, inter, glu, route, experts, ff,
                             route_input, stream);
    else if (act_type == RL_BF16)
        launch_swiglu<bf16_t>((const bf16_t*)gate_up, (bf16_t*)out, tokens, inter, glu, route, experts,
                              ff, route_input, stream);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// One-operand activations of a two-layer feed-forward, out = act(x):
//   kind 0: gelu in its tanh form, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))
//   kind 1: relu(z)^2
//   kind 2: tanh(z)
//   kind 3: gelu in its exact form, 0.5 z (1 + erf(z / sqrt(2)))
// With `route` (float32 [tokens, experts]) the first experts * ff columns of a row are the
// hidden units of `experts` experts side by side, and expert e's units are multiplied by
// route[t, e] (0 for an expert the token does not use); columns beyond (a shared expert's)
// pass with the activation alone, or with `route_shared` are multiplied by entry `experts` of the
// token's row of `route`, whose rows have route_width entries.
// --------------------------------------------------------------------------- //
__device__ inline float unary_act(float z, int kind) {
    if (kind == 1) {
        const float r = fmaxf(z, 0.f);
        return r * r;
    }
    if (kind == 2) return tanhf(z);
    if (kind == 3) return 0.5f * z * (1.f + erff(0.7071067811865476f * z));
    return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <typename T>
__global__ void unary_act_kernel(const T* __restrict__ x, T* __restrict__ out, size_t total, int cols,
                                 int kind, const float* __restrict__ route, int experts, int ff, int route_width,
                                 int route_shared) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        float v = unary_act(to_float(x[idx]), kind);
        if (route) {
            const size_t t = idx / cols;
            const int c = (int)(idx - t * cols);
            if (c < experts * ff || route_shared) v *= route[t * route_width + min(c / ff, experts)];
        }
        out[idx] = from_float<T>(v);
    }
}

// eight columns a thread: rows of a multiple of 8 columns, experts of a multiple of 8 hidden
// units, so that a group of eight belongs to one expert; `total` counts groups
template <typename T>
__global__ void unary_act_vec_kernel(const T* __restrict__ x, T* __restrict__ out, size_t total, int cols8,
                                     int kind, const float* __restrict__ route, int experts, int ff8, int route_width,
                                     int route_shared) {
    struct alignas(sizeof(T) * 8) Pack {
        T v[8];
    };
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const Pack in = reinterpret_cast<const Pack*>(x)[idx];
        float factor = 1.f;
        if (route) {
            const size_t t = idx / cols8;
            const int c = (int)(idx - t * cols8);
            if (c < experts * ff8 || route_shared) factor = route[t * route_width + min(c / ff8, experts)];
        }
        Pack o;
#pragma unroll
        for (int j = 0; j < 8; ++j) o.v[j] = from_float<T>(unary_act(to_float(in.v[j]), kind) * factor);
        reinterpret_cast<Pack*>(out)[idx] = o;
    }
}

extern "C" int rl_unary_act(const void* x, void* out, int tokens, int cols, int kind, const float* route,
                            int experts, int ff, int route_width, int route_shared, int act_type,
                            hipStream_t stream) {
    if (tokens <= 0 || cols <= 0) return RL_OK;
    if (kind < 0 || kind > 3) return RL_ERR_ARG;
    if (route && (experts < 1 || ff < 1 || (long)experts * ff > cols || route_width < experts + (route_shared ? 1 : 0)))
        return RL_ERR_ARG;
    if (act_type != RL_F32 && act_type != RL_BF16) return RL_ERR_ARG;
    const bool vec = cols % 8 == 0 && (!route || ff % 8 == 0);
    const size_t total = (size_t)tokens * cols / (vec ? 8 : 1);
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    dim3 grid((unsigned)blocks), block(256);
    if (vec && act_type == RL_F32)
        hipLaunchKernelGGL(unary_act_vec_kernel<float>, grid, block, 0, stream, (const float*)x, (float*)out, total,
                           cols / 8, kind, route, experts, ff / 8, route_width, route_shared);
    else if (vec)
        hipLaunchKernelGGL(unary_act_vec_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)x, (bf16_t*)out,
                           total, cols / 8, kind, route, experts, ff / 8, route_width, route_shared);
    else if (act_type == RL_F32)
        hipLaunchKernelGGL(unary_act_kernel<float>, grid, block, 0, stream, (const float*)x, (float*)out, total,
                           cols, kind, route, experts, ff, route_width, route_shared);
    else
        hipLaunchKernelGGL(unary_act_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)x, (bf16_t*)out,
                           total, cols, kind, route, experts, ff, route_width, route_shared);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// Router of a mixture of experts, one thread a token, float32 throughout:
//   s = softmax(z) over all experts; the `top` largest are chosen (the lower index wins a tie);
//   route[t, e] = s_e / (sum of the chosen s + 1e-20) * scale for a chosen expert, else 0.
// z is overwritten by route.
// With `sigmoid` scores, s = 1 / (1 + exp(-z)) and a chosen expert's weight is s_e * scale as it
// is: the chosen scores are not divided by their sum.
// --------------------------------------------------------------------------- //
#define ROUTE_MAX_EXPERTS 1024
// (a chosen expert's score is marked by its sign: scores are exponentials, never below +0)
__device__ inline void route_row(float* __restrict__ row, float* __restrict__ dst, int experts, int top, float scale,
                                 int sigmoid = 0) {
    if (sigmoid) {
        // The largest scores are the largest logits, and the logits are what is compared: two
        // scores that round to the same float32 (both 1 beyond a logit of 17) still differ there.
        // dst (not row: the router kernel's logits lie in LDS) holds 0 until an expert is chosen.
        for (int e = 0; e < experts; ++e) dst[e] = 0.f;
        for (int k = 0; k < top; ++k) {
            int best = -1;
            float best_z = -INFINITY;
            for (int e = 0; e < experts; ++e) {
                if (dst[e] == 0.f && row[e] > best_z) {
                    best_z = row[e];
                    best = e;
                }
            }
            if (best < 0) break;
            dst[best] = scale / (1.f + expf(-best_z));
        }
        return;
    }
    float m = -INFINITY;
    for (int e = 0; e < experts; ++e) m = fmaxf(m, row[e]);
    float total = 0.f;
    for (int e = 0; e < experts; ++e) {
        const float p = expf(row[e] - m);
        row[e] = p;
        total += p;
    }
    float sum = 0.f;
    for (int k = 0; k < top; ++k) {
        int best = 0;
        float best_s = -1.f;
        for (int e = 0; e < experts; ++e) {
            const float p = row[e];
            if (!signbit(p) && p > best_s) {
                best_s = p;
                best = e;
            }
        }
        row[best] = -best_s;
        sum += best_s / total;
    }
    const float inv = scale / (sum + 1e-20f);
    for (int e = 0; e < experts; ++e) {
        const float p = row[e];
        dst[e] = signbit(p) ? -p / total * inv : 0.f;
    }
}

__global__ void route_kernel(float* __restrict__ z, int tokens, int experts, int top, float scale) {
    const int t = blockIdx.x * blockDim.x + threadIdx.x;
    if (t >= tokens) return;
    route_row(z + (size_t)t * experts, z + (size_t)t * experts, experts, top, scale);
}

extern "C" int rl_route(float* z, int tokens, int experts, int top, float scale, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (experts < 1 || experts > ROUTE_MAX_EXPERTS || top < 1 || top > experts) return RL_ERR_ARG;
    hipLaunchKernelGGL(route_kernel, dim3((tokens + 63) / 64), dim3(64), 0, stream, z, tokens, experts, top, scale);
    return rl_launch_status();
}

// The router's product and the weights in one kernel: a wave takes a token, computes
// z_e = w[e] . x[t] in float32 for every expert (lanes stride the row, their sums are folded by
// the wave: one order of summation per token whatever else is in the step), and its first
// lane turns the logits into weights.  x may be bfloat16 or float32; w is float32; `bias`
// (optional, float32, one number an expert) is added to the logits.
template <typename T>
__global__ __launch_bounds__(256) void router_kernel(const T* __restrict__ x, const float* __restrict__ w,
                                                     float* __restrict__ route, int tokens, int k, int experts,
                                                     int top, float scale, const float* __restrict__ bias,
                                                     int sigmoid) {
    extern __shared__ float s_logits[];  // [4][experts]
    const int lane = threadIdx.x & (RL_WAVE - 1);
    const int wave = threadIdx.x / RL_WAVE;
    const int t = blockIdx.x * 4 + wave;
    if (t >= tokens) return;  // whole waves leave; nothing below waits for another wave
    float* z = s_logits + (size_t)wave * experts;
    const T* xr = x + (size_t)t * k;
    // eight experts at a time, so that a chunk of x is read once for eight rows of w and the
    // loads of an iteration do not wait for each other
    for (int e0 = 0; e0 < experts; e0 += 8) {
        float acc[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = 0.f;
        const int ne = min(8, experts - e0);
        if (k % 4 == 0) {
            // (unrolled: the loads of four iterations are asked for together; a step of a few
            // tokens is all latency here)
#pragma unroll 4
            for (int i = 4 * lane; i < k; i += 4 * RL_WAVE) {
                const Vec4<T> xv = *reinterpret_cast<const Vec4<T>*>(xr + i);
                float4 wv[8];
#pragma unroll
                for (int j = 0; j < 8; ++j)
                    wv[j] = *reinterpret_cast<const float4*>(w + (size_t)(e0 + min(j, ne - 1)) * k + i);
                const float x0 = to_float(xv.v[0]), x1 = to_float(xv.v[1]), x2 = to_float(xv.v[2]),
                            x3 = to_float(xv.v[3]);
#pragma unroll
                for (int j = 0; j < 8; ++j)
                    acc[j] = fmaf(x3, wv[j].w, fmaf(x2, wv[j].z, fmaf(x1, wv[j].y, fmaf(x0, wv[j].x, acc[j]))));
            }
        } else {
            for (int i = lane; i < k; i += RL_WAVE) {
                const float xv = to_float(xr[i]);
#pragma unroll
                for (int j = 0; j < 8; ++j) acc[j] = fmaf(xv, w[(size_t)(e0 + min(j, ne - 1)) * k + i], acc[j]);
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float sum = wave_sum(acc[j]);
            if (lane == 0 && j < ne) z[e0 + j] = bias ? sum + bias[e0 + j] : sum;
        }
    }
    if (lane == 0) route_row(z, route + (size_t)t * experts, experts, top, scale, sigmoid);
}

extern "C" int rl_router(const void* x, const float* w, float* route, int tokens, int k, int experts, int top,
                         float scale, const float* bias, int sigmoid, int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (k < 1 || experts < 1 || experts > ROUTE_MAX_EXPERTS || top < 1 || top > experts) return RL_ERR_ARG;
    dim3 grid((tokens + 3) / 4), block(256);
    const size_t lds = (size_t)4 * experts * sizeof(float);
    if (act_type == RL_F32)
        hipLaunchKernelGGL(router_kernel<float>, grid, block, lds, stream, (const float*)x, w, route, tokens, k,
                           experts, top, scale, bias, sigmoid);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(router_kernel<bf16_t>, grid, block, lds, stream, (const bf16_t*)x, w, route, tokens, k,
                           experts, top, scale, bias, sigmoid);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// cast between float32 and bfloat16 (either direction, or a copy)
// --------------------------------------------------------------------------- //
template <typename S, typename D>
__global__ void cast_kernel(const S* __restrict__ src, D* __restrict__ dst, size_t total) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) dst[idx] = from_float<D>(to_float(src[idx]));
}

extern "C" int rl_cast(const void* src, int src_type, void* dst, int dst_type, size_t total,
                       hipStream_t stream) {
    if (total == 0) return RL_OK;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    dim3 grid((unsigned)blocks), block(256);
    if (src_type == RL_F32 && dst_type == RL_BF16)
        hipLaunchKernelGGL((cast_kernel<float, bf16_t>), grid, block, 0, stream,
                           (const float*)src, (bf16_t*)dst, total);
    else if (src_type == RL_BF16 && dst_type == RL_F32)
        hipLaunchKernelGGL((cast_kernel<bf16_t, float>), grid, block, 0, stream,
                           (const bf16_t*)src, (float*)dst, total);
    else if (src_type == RL_F32 && dst_type == RL_F32)
        hipLaunchKernelGGL((cast_kernel<float, float>), grid, block, 0, stream,
                           (const float*)src, (float*)dst, total);
    else if (src_type == RL_BF16 && dst_type == RL_BF16)
        hipLaunchKernelGGL((cast_kernel<bf16_t, bf16_t>), grid, block, 0, stream,
                           (const bf16_t*)src, (bf16_t*)dst, total);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// bias of a product: y[r, c] += bias[c], the sum rounded once to y's type
// (rapid_llm/modules/linear.py adds the bias inside F.linear; Qwen3 has none, other
// architectures' projections do)
// --------------------------------------------------------------------------- //
template <typename T>
__global__ void add_bias_kernel(T* __restrict__ y, const float* __restrict__ bias, size_t total,
                                int cols) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) y[idx] = from_float<T>(to_float(y[idx]) + bias[idx % cols]);
}

extern "C" int rl_add_bias(void* y, const float* bias, int rows, int cols, int act_type,
                           hipStream_t stream) {
    if (rows <= 0 || cols <= 0) return RL_OK;
    const size_t total = (size_t)rows * cols;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    dim3 grid((unsigned)blocks), block(256);
    if (act_type == RL_F32)
        hipLaunchKernelGGL(add_bias_kernel<float>, grid, block, 0, stream, (float*)y, bias, total, cols);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(add_bias_kernel<bf16_t>, grid, block, 0, stream, (bf16_t*)y, bias, total, cols);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// residual[r, :] += first[r, :] + row[:] (float32, in place; either may be null): what a pass over
// a span of layers begins with, the embedding's output once more and a vector of the pass
// --------------------------------------------------------------------------- //
__global__ void stream_add_kernel(float* __restrict__ residual, const float* __restrict__ first,
                                  const float* __restrict__ row, size_t total, int hidden) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        float v = residual[idx];
        if (first) v += first[idx];
        if (row) v += row[idx % hidden];
        residual[idx] = v;
    }
}

__global__ void stream_add_vec_kernel(float4* __restrict__ residual, const float4* __restrict__ first,
                                      const float4* __restrict__ row, size_t total, int hidden4) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        float4 v = residual[idx];
        if (first) {
            const float4 f = first[idx];
            v.x += f.x; v.y += f.y; v.z += f.z; v.w += f.w;
        }
        if (row) {
            const float4 w = row[idx % hidden4];
            v.x += w.x; v.y += w.y; v.z += w.z; v.w += w.w;
        }
        residual[idx] = v;
    }
}

extern "C" int rl_stream_add(float* residual, const float* first, const float* row, int tokens, int hidden,
                             hipStream_t stream) {
    if (tokens <= 0 || hidden <= 0 || (!first && !row)) return RL_OK;
    const bool vec = hidden % 4 == 0;
    const size_t total = (size_t)tokens * hidden / (vec ? 4 : 1);
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    if (vec)
        hipLaunchKernelGGL(stream_add_vec_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, (float4*)residual,
                           (const float4*)first, (const float4*)row, total, hidden / 4);
    else
        hipLaunchKernelGGL(stream_add_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, residual, first, row,
                           total, hidden);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// gate of a head: y[t, h, :] *= sigmoid(packed[t, gate_col + h]), one number a head, read
// from a column of the row that the mixer's packed projection wrote
// --------------------------------------------------------------------------- //
template <typename T>
__global__ void head_gate_kernel(T* __restrict__ y, const T* __restrict__ packed, int row_width,
                                 int gate_col, int heads, int d, size_t total) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    const size_t per_token = (size_t)heads * d;
    for (; idx < total; idx += step) {
        const size_t t = idx / per_token;
        const int h = (int)((idx - t * per_token) / d);
        const float g = to_float(packed[t * row_width + gate_col + h]);
        y[idx] = from_float<T>(to_float(y[idx]) / (1.f + expf(-g)));
    }
}

extern "C" int rl_head_gate(void* y, const void* packed, int row_width, int gate_col, int tokens,
                            int heads, int d, int act_type, hipStream_t stream) {
    if (tokens <= 0 || heads <= 0 || d <= 0) return RL_OK;
    if (gate_col < 0 || gate_col + heads > row_width) return RL_ERR_ARG;
    const size_t total = (size_t)tokens * heads * d;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    dim3 grid((unsigned)blocks), block(256);
    if (act_type == RL_F32)
        hipLaunchKernelGGL(head_gate_kernel<float>, grid, block, 0, stream, (float*)y, (const float*)packed,
                           row_width, gate_col, heads, d, total);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(head_gate_kernel<bf16_t>, grid, block, 0, stream, (bf16_t*)y, (const bf16_t*)packed,
                           row_width, gate_col, heads, d, total);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// rotation tables: cos/sin[p, i] of the float32 product p * inv_freq[i]
// rapid_llm/modules/rotary_embedding.py:194-202 (float32 outer product, then cos/sin)
// --------------------------------------------------------------------------- //
__global__ void rope_table_kernel(const float* __restrict__ inv_freq, float* __restrict__ cos_out,
                                  float* __restrict__ sin_out, int half, size_t total) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const size_t p = idx / half;
        const int i = (int)(idx - p * half);
        const float ang = (float)p * inv_freq[i];
        // the angle is the float32 product; its cosine and sine are taken in double so
        // that range reduction of large angles costs nothing in accuracy
        cos_out[idx] = (float)cos((double)ang);
        sin_out[idx] = (float)sin((double)ang);
    }
}

extern "C" int rl_rope_table(const float* inv_freq, float* cos_out, float* sin_out,
                             int positions, int half, hipStream_t stream) {
    const size_t total = (size_t)positions * half;
    if (total == 0) return RL_OK;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    hipLaunchKernelGGL(rope_table_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, inv_freq,
                       cos_out, sin_out, half, total);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// Fused per-head RMSNorm (optional) + rotation (optional) of q and k, and the write of k and v
// into the paged cache.  One wave per (token, head); a workgroup of four waves takes four
// heads of a token.
//
// qkv row layout: [q heads | k heads | v heads], heads adjacent (rapid_llm/modules/linear.py:
// 236-251).  Norm over head_dim before the rotation (rapid_llm/models/base.py:134-140).
// Rotation of a pair (x1, x2) by the position's angle of that pair: o1 = x1*c - x2*s,
// o2 = x2*c + x1*s (rapid_llm/kernels/ops/rope/rope_emb.py:47-82).  Which channels pair, and
// how many of a head's channels rotate, is the position encoding's to say: the first
// 2 * rotary_half channels rotate, pair p of them being channels (p, p + rotary_half) with the
// half-split pairing (the reference's) and (2p, 2p + 1) with the interleaved one; the channels
// beyond pass with the norm alone.  This kernel takes every such case; the vectorised ones
// below take the half-split rotation of the whole head.
//
// Cache layout of one layer, page p, kv head h:
//   keys   K[p][h][slot_in_page][d]      (row-major, d contiguous)
//   values V[p][h][dv][slot_in_page]     (transposed: the page's positions contiguous; a value
//                                         head has dv channels, which need not be d)
// A token at position pos of a request lies in page table[slot_of_request][pos / P] at
// slot_in_page = pos % P.
// --------------------------------------------------------------------------- //
// What may happen to the heads besides norm and rotation.
struct HeadPrep {
    const float* bias;  // the projection's, one entry a column of the packed row, added as heads are read
    // temp_coef != 0: finished queries are multiplied by 1 + temp_coef * ln(floor((pos + 1) / temp_every) + 1)
    float temp_coef, temp_every;
    int norm_values;  // every value head is divided by its root mean square (eps inside the root, no weight)
};
__device__ inline float query_temperature(const HeadPrep& hp, int pos) {
    // (the division of two integers below 2^24 rounds to an integer only where it is one)
    return 1.f + hp.temp_coef * logf(floorf((float)(pos + 1) / hp.temp_every) + 1.f);
}

// 1 / (root mean square) of a value head, in every one of (at least) 16 lanes of a wave that read the
// same head: each row of 16 lanes forms the sum, in the order of the tile kernel below
template <typename T>
__device__ inline float value_factor(const T* __restrict__ xv, const float* __restrict__ vb, int dv, float eps) {
    float ss = 0.f;
    for (int i = threadIdx.x % 16; i < dv; i += 16) {
        const float v = to_float(xv[i]) + (vb ? vb[i] : 0.f);
        ss += v * v;
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o, RL_WAVE);
    return rsqrtf(ss / (float)dv + eps);
}

template <typename T>
__global__ void qknorm_rope_kvwrite_kernel(
    const T* __restrict__ qkv, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const float* __restrict__ q_norm_w,
    const float* __restrict__ k_norm_w, const float* __restrict__ cos_tab,
    const float* __restrict__ sin_tab, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int nq, int nkv, int d, int rotary_half, int interleaved, float eps,
    int write_cache, int write_values, int head0, int row_width, int v_col0, int dv, HeadPrep hp) {
    const int t = blockIdx.x;
    const int lane = threadIdx.x & (RL_WAVE - 1);
    const int wave = threadIdx.x / RL_WAVE;
    const int nwaves = blockDim.x / RL_WAVE;
    const int half = (d + 1) / 2;  // of an odd size the last pair holds one channel
    const int pos = positions[t];
    const int total_heads = nq + 2 * nkv;
    const T* row = qkv + (size_t)t * row_width;

    size_t page = 0;
    int off = 0;
    if (write_cache) {
        page = (size_t)block_table[(size_t)token_slot[t] * table_stride + pos / page_size];
        off = pos % page_size;
    }

    // head0: the first head to work on (the number of query heads where the attention kernels
    // finish the queries themselves)
    for (int head = head0 + blockIdx.y * nwaves + wave; head < total_heads; head += nwaves * gridDim.y) {
        const T* x = row + (size_t)head * d;
        if (head >= nq + nkv) {
            // value head: copy into the transposed page (unless the tile kernel below does it)
            if (!write_cache || !write_values) continue;
            const int h = head - nq - nkv;
            const T* xv = row + v_col0 + (size_t)h * dv;  // where the row keeps this value head
            T* dst = v_cache + ((page * nkv + h) * dv) * page_size + off;
            const float* vb = hp.bias ? hp.bias + v_col0 + (size_t)h * dv : nullptr;
            const float factor = hp.norm_values ? value_factor(xv, vb, dv, eps) : 1.f;
            for (int i = lane; i < dv; i += RL_WAVE)
                dst[(size_t)i * page_size] = from_float<T>((to_float(xv[i]) + (vb ? vb[i] : 0.f)) * factor);
            continue;
        }
        const bool is_q = head < nq;
        if (!is_q && !write_cache) continue;
        const float* w = is_q ? q_norm_w : k_norm_w;
        // lane handles the pairs p = lane, lane + 64 (half <= 128) of channels (e1, e2): the
        // pairs that rotate first, as the pairing says, then the channels beyond two by two
        const int rot = cos_tab ? rotary_half : 0;
        int e1[2], e2[2];
        float x1[2], x2[2];
        float ss = 0.f;
#pragma unroll
        for (int r = 0; r < 2; ++r) {
            const int p = lane + r * RL_WAVE;
            const bool split = p < rot && !interleaved;
            e1[r] = split ? p : 2 * p;
            e2[r] = split ? p + rot : 2 * p + 1;
            x1[r] = 0.f;
            x2[r] = 0.f;
            if (p < half) {
                x1[r] = to_float(x[e1[r]]);
                if (e2[r] < d) x2[r] = to_float(x[e2[r]]);
                if (hp.bias) {  // the projection's bias, added here instead of by a kernel of its own
                    x1[r] += hp.bias[(size_t)head * d + e1[r]];
                    if (e2[r] < d) x2[r] += hp.bias[(size_t)head * d + e2[r]];
                }
                ss += x1[r] * x1[r] + x2[r] * x2[r];
            }
        }
        float rrms = 1.f;
        if (w) {
            ss = wave_sum(ss);
            rrms = rsqrtf(ss / (float)d + eps);
        }
        const float temp = (is_q && hp.temp_coef != 0.f) ? query_temperature(hp, pos) : 1.f;
        T* dst;
        if (is_q)
            dst = q_out + ((size_t)t * nq + head) * d;
        else
            dst = k_cache + ((page * nkv + (head - nq)) * page_size + off) * d;
#pragma unroll
        for (int r = 0; r < 2; ++r) {
            const int p = lane + r * RL_WAVE;
            if (p < half) {
                float a = x1[r], b = x2[r];
                if (w) {
                    a = a * rrms * w[e1[r]];
                    if (e2[r] < d) b = b * rrms * w[e2[r]];
                }
                if (p < rot) {
                    const float c = cos_tab[(size_t)pos * rotary_half + p];
                    const float s = sin_tab[(size_t)pos * rotary_half + p];
                    const float ra = a * c - b * s;
                    const float rb = b * c + a * s;
                    a = ra;
                    b = rb;
                }
                dst[e1[r]] = from_float<T>(a * temp);
                if (e2[r] < d) dst[e2[r]] = from_float<T>(b * temp);
            }
        }
    }
}

// The same with four consecutive channels of each half per lane: LPH lanes (16 for heads up to
// 128, else 32) take one head, a wave takes 64 / LPH heads, and every load and store moves 8
// or 16 bytes.  Needs d % 8 == 0.
template <typename T, int LPH>
__device__ inline void qknorm_rope_kvwrite_vec(
    int t, int head_group, const T* __restrict__ qkv, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const float* __restrict__ q_norm_w,
    const float* __restrict__ k_norm_w, const float* __restrict__ cos_tab,
    const float* __restrict__ sin_tab, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int nq, int nkv, int d, float eps, int write_cache, int write_values, int head0,
    int row_width, int v_col0, int dv, HeadPrep hp) {
    constexpr int HPW = RL_WAVE / LPH;  // heads per wave
    const int lane = threadIdx.x & (RL_WAVE - 1);
    const int wave = threadIdx.x / RL_WAVE;
    const int sub = lane / LPH;  // which of the wave's heads
    const int li = lane % LPH;   // channels 4 li .. 4 li + 3 of each half
    const int half = d / 2;
    const int pos = positions[t];
    const int total_heads = nq + (write_values ? 2 * nkv : nkv);
    const T* row = qkv + (size_t)t * row_width;
    size_t page = 0;
    int off = 0;
    if (write_cache) {
        page = (size_t)block_table[(size_t)token_slot[t] * table_stride + pos / page_size];
        off = pos % page_size;
    }
    const int head = head0 + (head_group * (blockDim.x / RL_WAVE) + wave) * HPW + sub;
    if (head >= total_heads) return;  // whole groups of LPH lanes leave together
    const T* x = row + (size_t)head * d;
    const bool active = 4 * li < half;
    if (head >= nq + nkv) {
        if (!write_cache) return;
        const int h = head - nq - nkv;
        const T* xv = row + v_col0 + (size_t)h * dv;
        T* dst = v_cache + ((page * nkv + h) * dv) * page_size + off;
        const float* vb = hp.bias ? hp.bias + v_col0 + (size_t)h * dv : nullptr;
        const float factor = hp.norm_values ? value_factor(xv, vb, dv, eps) : 1.f;
        for (int i = li; i < dv; i += LPH)
            dst[(size_t)i * page_size] = from_float<T>((to_float(xv[i]) + (vb ? vb[i] : 0.f)) * factor);
        return;
    }
    const bool is_q = head < nq;
    if (!is_q && !write_cache) return;
    const float* w = is_q ? q_norm_w : k_norm_w;
    float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
    float ss = 0.f;
    if (active) {
        const Vec4<T> va = *reinterpret_cast<const Vec4<T>*>(x + 4 * li);
        const Vec4<T> vb = *reinterpret_cast<const Vec4<T>*>(x + half + 4 * li);
        Vec4<float> ba = {}, bb = {};
        if (hp.bias) {
            ba = *reinterpret_cast<const Vec4<float>*>(hp.bias + (size_t)head * d + 4 * li);
            bb = *reinterpret_cast<const Vec4<float>*>(hp.bias + (size_t)head * d + half + 4 * li);
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            a[k] = to_float(va.v[k]) + ba.v[k];
            b[k] = to_float(vb.v[k]) + bb.v[k];
            ss += a[k] * a[k] + b[k] * b[k];
        }
    }
    if (w) {
        // sum over the LPH lanes of the head (a power of two, aligned in the wave)
#pragma unroll
        for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, RL_WAVE);
        const float rrms = rsqrtf(ss / (float)d + eps);
        if (active) {
            const float4 wa = *reinterpret_cast<const float4*>(w + 4 * li);
            const float4 wb = *reinterpret_cast<const float4*>(w + half + 4 * li);
            a[0] *= rrms * wa.x; a[1] *= rrms * wa.y; a[2] *= rrms * wa.z; a[3] *= rrms * wa.w;
            b[0] *= rrms * wb.x; b[1] *= rrms * wb.y; b[2] *= rrms * wb.z; b[3] *= rrms * wb.w;
        }
    }
    if (!active) return;
    if (cos_tab) {
        const float4 c4 = *reinterpret_cast<const float4*>(cos_tab + (size_t)pos * half + 4 * li);
        const float4 s4 = *reinterpret_cast<const float4*>(sin_tab + (size_t)pos * half + 4 * li);
        const float cs[4] = {c4.x, c4.y, c4.z, c4.w}, sn[4] = {s4.x, s4.y, s4.z, s4.w};
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const float ra = a[k] * cs[k] - b[k] * sn[k];
            b[k] = b[k] * cs[k] + a[k] * sn[k];
            a[k] = ra;
        }
    }
    T* dst = is_q ? q_out + ((size_t)t * nq + head) * d
                  : k_cache + ((page * nkv + (head - nq)) * page_size + off) * d;
    const float temp = (is_q && hp.temp_coef != 0.f) ? query_temperature(hp, pos) : 1.f;
    Vec4<T> oa, ob;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        oa.v[k] = from_float<T>(a[k] * temp);
        ob.v[k] = from_float<T>(b[k] * temp);
    }
    *reinterpret_cast<Vec4<T>*>(dst + 4 * li) = oa;
    *reinterpret_cast<Vec4<T>*>(dst + half + 4 * li) = ob;
}

template <typename T, int LPH>
__global__ __launch_bounds__(256) void qknorm_rope_kvwrite_vec_kernel(
    const T* __restrict__ qkv, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const float* __restrict__ q_norm_w,
    const float* __restrict__ k_norm_w, const float* __restrict__ cos_tab,
    const float* __restrict__ sin_tab, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int nq, int nkv, int d, float eps, int write_cache, int write_values, int head0,
    int row_width, int v_col0, int dv, HeadPrep hp) {
    qknorm_rope_kvwrite_vec<T, LPH>(blockIdx.x, blockIdx.y, qkv, q_out, k_cache, v_cache, q_norm_w, k_norm_w,
                                    cos_tab, sin_tab, positions, token_slot, block_table, table_stride,
                                    page_size, nq, nkv, d, eps, write_cache, write_values, head0, row_width,
                                    v_col0, dv, hp);
}

template <typename T>
static void launch_qknorm(const T* qkv, T* q_out, T* k_cache, T* v_cache, const float* q_norm_w,
                          const float* k_norm_w, const float* cos_tab, const float* sin_tab,
                          const int* positions, const int* token_slot, const int* block_table,
                          int table_stride, int page_size, int tokens, int nq, int nkv, int d,
                          int rotary_half, int interleaved, float eps, int write_cache,
                          int write_values, int head0, int row_width, int v_col0, int dv, HeadPrep hp, hipStream_t stream) {
    const int total_heads = nq + (write_values ? 2 * nkv : nkv) - head0;  // heads to work on
    // the vectorised kernel: head sizes in steps of 8, the half-split rotation of the whole head
    if (d % 8 == 0 && (!cos_tab || (rotary_half == d / 2 && !interleaved))) {
        const int lph = d <= 128 ? 16 : 32;
        const int heads_per_block = 4 * (RL_WAVE / lph);
        const int groups = (total_heads + heads_per_block - 1) / heads_per_block;
        dim3 grid(tokens, groups), block(256);
        if (lph == 16)
            hipLaunchKernelGGL((qknorm_rope_kvwrite_vec_kernel<T, 16>), grid, block, 0, stream, qkv,
                               q_out, k_cache, v_cache, q_norm_w, k_norm_w, cos_tab, sin_tab,
                               positions, token_slot, block_table, table_stride, page_size, nq, nkv,
                               d, eps, write_cache, write_values, head0, row_width, v_col0, dv, hp);
        else
            hipLaunchKernelGGL((qknorm_rope_kvwrite_vec_kernel<T, 32>), grid, block, 0, stream, qkv,
                               q_out, k_cache, v_cache, q_norm_w, k_norm_w, cos_tab, sin_tab,
                               positions, token_slot, block_table, table_stride, page_size, nq, nkv,
                               d, eps, write_cache, write_values, head0, row_width, v_col0, dv, hp);
        return;
    }
    const int head_groups = (total_heads + 3) / 4;
    dim3 grid(tokens, head_groups > 65535 ? 65535 : head_groups), block(256);
    hipLaunchKernelGGL(qknorm_rope_kvwrite_kernel<T>, grid, block, 0, stream, qkv, q_out, k_cache,
                       v_cache, q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot,
                       block_table, table_stride, page_size, nq, nkv, d, rotary_half, interleaved, eps,
                       write_cache, write_values, head0, row_width, v_col0, dv, hp);
}

// Values of 16 consecutive tokens of the batch and one kv head, written by one workgroup.
// The cache stores values transposed, V[page][head][channel][slot]: the sixteen slots of a
// channel are one 32-byte row (at a page of 16), and consecutive tokens of a request fill
// consecutive slots of it.  Written token by token those rows are completed by sixteen
// different workgroups, 2 bytes at a time; here a thread writes the four slots of four
// consecutive tokens at once where they line up, and the four threads of a row sit in
// adjacent lanes.
#define VT_TOKENS 16

template <typename T>
__device__ inline void v_tile_write(
    int tile, int h, const T* __restrict__ qkv, T* __restrict__ v_cache, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int tokens, int nq, int nkv, int d, int row_width, int v_col0, int dv, float eps, HeadPrep hp) {
    __shared__ float vt[VT_TOKENS][256 + 8];
    __shared__ int s_page[VT_TOKENS];
    __shared__ int s_off[VT_TOKENS];
    __shared__ float s_factor[VT_TOKENS];
    const int t0 = tile * VT_TOKENS;
    if (threadIdx.x < VT_TOKENS) {
        const int t = t0 + threadIdx.x;
        int page = -1, off = 0;
        if (t < tokens) {
            const int pos = positions[t];
            page = block_table[(size_t)token_slot[t] * table_stride + pos / page_size];
            off = pos % page_size;
        }
        s_page[threadIdx.x] = page;
        s_off[threadIdx.x] = off;
    }
    for (int idx = threadIdx.x; idx < VT_TOKENS * dv; idx += 256) {
        const int i = idx / dv, c = idx - i * dv;
        if (t0 + i < tokens) {
            const float v = to_float(qkv[(size_t)(t0 + i) * row_width + v_col0 + (size_t)h * dv + c]);
            vt[i][c] = hp.bias ? v + hp.bias[v_col0 + (size_t)h * dv + c] : v;
        }
    }
    __syncthreads();
    if (hp.norm_values) {  // sixteen threads a token
        const int i = threadIdx.x / 16;
        float ss = 0.f;
        if (t0 + i < tokens)
            for (int c = threadIdx.x % 16; c < dv; c += 16) ss += vt[i][c] * vt[i][c];
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o, RL_WAVE);
        if (threadIdx.x % 16 == 0) s_factor[i] = rsqrtf(ss / (float)dv + eps);
        __syncthreads();
    }
    for (int idx = threadIdx.x; idx < 4 * dv; idx += 256) {
        const int quarter = idx & 3, c = idx >> 2;
        const int i0 = 4 * quarter;
        const int page = s_page[i0], off = s_off[i0];
        bool lined_up = page >= 0 && (off & 3) == 0 && (page_size & 3) == 0;
#pragma unroll
        for (int k = 1; k < 4; ++k)
            lined_up = lined_up && s_page[i0 + k] == page && s_off[i0 + k] == off + k;
        if (lined_up) {
            Vec4<T> v;
#pragma unroll
            for (int k = 0; k < 4; ++k)
                v.v[k] = from_float<T>(hp.norm_values ? vt[i0 + k][c] * s_factor[i0 + k] : vt[i0 + k][c]);
            *reinterpret_cast<Vec4<T>*>(v_cache + (((size_t)page * nkv + h) * dv + c) * page_size + off) = v;
        } else {
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const int pg = s_page[i0 + k];
                if (pg >= 0)
                    v_cache[(((size_t)pg * nkv + h) * dv + c) * page_size + s_off[i0 + k]] =
                        from_float<T>(hp.norm_values ? vt[i0 + k][c] * s_factor[i0 + k] : vt[i0 + k][c]);
            }
        }
    }
}

// One launch for a step of many tokens: the first tokens * head_groups workgroups norm, rotate
// and write the query and key heads of one token each, the rest write the values of 16 tokens
// and one kv head each.  A workgroup is wholly one or the other.
template <typename T, int LPH>
__global__ __launch_bounds__(256) void qkv_prepare_kernel(
    const T* __restrict__ qkv, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const float* __restrict__ q_norm_w,
    const float* __restrict__ k_norm_w, const float* __restrict__ cos_tab,
    const float* __restrict__ sin_tab, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int tokens, int head_groups, int nq, int nkv, int d, float eps, int head0,
    int row_width, int v_col0, int dv, HeadPrep hp) {
    const int qk_blocks = tokens * head_groups;
    if ((int)blockIdx.x < qk_blocks) {
        qknorm_rope_kvwrite_vec<T, LPH>(blockIdx.x / head_groups, blockIdx.x % head_groups, qkv, q_out, k_cache,
                                        v_cache, q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot,
                                        block_table, table_stride, page_size, nq, nkv, d, eps, 1, 0, head0,
                                        row_width, v_col0, dv, hp);
    } else {
        const int b = blockIdx.x - qk_blocks;
        v_tile_write<T>(b / nkv, b % nkv, qkv, v_cache, positions, token_slot, block_table, table_stride,
                        page_size, tokens, nq, nkv, d, row_width, v_col0, dv, eps, hp);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void v_tile_write_kernel(
    const T* __restrict__ qkv, T* __restrict__ v_cache, const int* __restrict__ positions,
    const int* __restrict__ token_slot, const int* __restrict__ block_table, int table_stride,
    int page_size, int tokens, int nq, int nkv, int d, int row_width, int v_col0, int dv, float eps, HeadPrep hp) {
    v_tile_write<T>(blockIdx.x, blockIdx.y, qkv, v_cache, positions, token_slot, block_table, table_stride,
                    page_size, tokens, nq, nkv, d, row_width, v_col0, dv, eps, hp);
}

// true if it launched: head sizes in steps of 8, and a grid that fits
template <typename T>
static bool launch_qkv_prepare(const T* qkv, T* q_out, T* k_cache, T* v_cache, const float* q_norm_w,
                               const float* k_norm_w, const float* cos_tab, const float* sin_tab,
                               const int* positions, const int* token_slot, const int* block_table,
                               int table_stride, int page_size, int tokens, int nq, int nkv, int d,
                               float eps, int head0, int row_width, int v_col0, int dv, HeadPrep hp, hipStream_t stream) {
    if (d % 8) return false;
    const int lph = d <= 128 ? 16 : 32;
    const int heads_per_block = 4 * (RL_WAVE / lph);
    const int head_groups = (nq + nkv - head0 + heads_per_block - 1) / heads_per_block;
    const long blocks = (long)tokens * head_groups + (long)((tokens + VT_TOKENS - 1) / VT_TOKENS) * nkv;
    if (blocks > 0x7fffffffL) return false;
    dim3 grid((unsigned)blocks), block(256);
    if (lph == 16)
        hipLaunchKernelGGL((qkv_prepare_kernel<T, 16>), grid, block, 0, stream, qkv, q_out, k_cache, v_cache,
                           q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot, block_table,
                           table_stride, page_size, tokens, head_groups, nq, nkv, d, eps, head0, row_width,
                           v_col0, dv, hp);
    else
        hipLaunchKernelGGL((qkv_prepare_kernel<T, 32>), grid, block, 0, stream, qkv, q_out, k_cache, v_cache,
                           q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot, block_table,
                           table_stride, page_size, tokens, head_groups, nq, nkv, d, eps, head0, row_width,
                           v_col0, dv, hp);
    return true;
}

extern "C" int rl_qknorm_rope_kvwrite(const void* qkv, void* q_out, void* k_cache, void* v_cache,
                                      const float* q_norm_w, const float* k_norm_w,
                                      const float* cos_tab, const float* sin_tab,
                                      const int* positions, const int* token_slot,
                                      const int* block_table, int table_stride, int page_size,
                                      int tokens, int nq, int nkv, int d, int rotary_half,
                                      int interleaved, float eps, int write_cache, int row_width, int v_col0, int dv,
                                      const float* bias, float temp_coef, float temp_every, int norm_values,
                                      int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (temp_coef != 0.f && !(temp_every > 0.f && q_out)) return RL_ERR_ARG;
    const HeadPrep hp = {bias, temp_coef, temp_every, norm_values};
    if (d < 1 || (d % 2 && cos_tab) || d > 256) return RL_ERR_ARG;
    // the packed row: query heads from column 0, key heads behind them, the nkv value heads of dv
    // channels from column v_col0 on ((nq + nkv) * d: behind the keys; nq * d: the values are the
    // unrotated keys)
    if (dv < 1 || dv > 256 || v_col0 < 0 || row_width < (nq + nkv) * d || v_col0 + nkv * dv > row_width)
        return RL_ERR_ARG;
    // q_out null: the attention kernels finish the query heads themselves, and the work here
    // starts at the first key head
    const int head0 = q_out ? 0 : nq;
    if (!q_out && !write_cache) return RL_OK;  // nothing to write at all
    // the first 2 * rotary_half channels of a head rotate: at least one pair, at most all
    if (cos_tab && (rotary_half < 1 || rotary_half > d / 2)) return RL_ERR_ARG;
    const bool whole_split = !cos_tab || (rotary_half == d / 2 && !interleaved);
    // with enough tokens the values go through the tile kernel, and the per-head kernel
    // covers the query and key heads only
    const int tile_values = write_cache && tokens >= 8 && nkv <= 65535;
    if ((long)nq + 2 * nkv > 65535 * 4) return RL_ERR_ARG;
    dim3 block(256);
    dim3 vgrid((tokens + VT_TOKENS - 1) / VT_TOKENS, nkv);
    if (tile_values && whole_split && act_type == RL_F32 &&
        launch_qkv_prepare<float>((const float*)qkv, (float*)q_out, (float*)k_cache, (float*)v_cache, q_norm_w,
                                  k_norm_w, cos_tab, sin_tab, positions, token_slot, block_table,
                                  table_stride, page_size, tokens, nq, nkv, d, eps, head0, row_width, v_col0, dv, hp,
                                  stream))
        return rl_launch_status();
    if (tile_values && whole_split && act_type == RL_BF16 &&
        launch_qkv_prepare<bf16_t>((const bf16_t*)qkv, (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache,
                                   q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot, block_table,
                                   table_stride, page_size, tokens, nq, nkv, d, eps, head0, row_width, v_col0, dv, hp,
                                   stream))
        return rl_launch_status();
    if (act_type == RL_F32) {
        launch_qknorm<float>((const float*)qkv, (float*)q_out, (float*)k_cache, (float*)v_cache,
                             q_norm_w, k_norm_w, cos_tab, sin_tab, positions, token_slot,
                             block_table, table_stride, page_size, tokens, nq, nkv, d, rotary_half,
                             interleaved, eps, write_cache, !tile_values, head0, row_width, v_col0, dv, hp, stream);
        if (tile_values)
            hipLaunchKernelGGL(v_tile_write_kernel<float>, vgrid, block, 0, stream,
                               (const float*)qkv, (float*)v_cache, positions, token_slot,
                               block_table, table_stride, page_size, tokens, nq, nkv, d, row_width, v_col0, dv, eps, hp);
    } else if (act_type == RL_BF16) {
        launch_qknorm<bf16_t>((const bf16_t*)qkv, (bf16_t*)q_out, (bf16_t*)k_cache,
                              (bf16_t*)v_cache, q_norm_w, k_norm_w, cos_tab, sin_tab, positions,
                              token_slot, block_table, table_stride, page_size, tokens, nq, nkv, d,
                              rotary_half, interleaved, eps, write_cache, !tile_values, head0, row_width,
                              v_col0, dv, hp, stream);
        if (tile_values)
            hipLaunchKernelGGL(v_tile_write_kernel<bf16_t>, vgrid, block, 0, stream,
                               (const bf16_t*)qkv, (bf16_t*)v_cache, positions, token_slot,
                               block_table, table_stride, page_size, tokens, nq, nkv, d, row_width, v_col0, dv, eps, hp);
    } else {
        return RL_ERR_ARG;
    }
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// order[r] = the single-token request with the r-th longest context of the step: request i's
// last position is positions[seq_token ? seq_token[i] : i]; equal lengths keep their order.
// Every thread counts the requests that come before its own (n^2 comparisons through LDS:
// a step has hundreds of requests, not millions).  The decode attention hands its workgroups
// out in this order.
// --------------------------------------------------------------------------- //
__global__ __launch_bounds__(256) void order_by_length_kernel(const int* __restrict__ positions,
                                                              const int* __restrict__ seq_token,
                                                              int n, int* __restrict__ order) {
    __shared__ __attribute__((aligned(16))) int keys[256];
    const int i = blockIdx.x * 256 + threadIdx.x;
    const int mine = i < n ? positions[seq_token ? seq_token[i] : i] : 0;
    int rank = 0;
    for (int base = 0; base < n; base += 256) {  // the same trips for every thread
        const int j = base + threadIdx.x;
        __syncthreads();
        // beyond the last request: shorter than any (positions are never negative)
        keys[threadIdx.x] = j < n ? positions[seq_token ? seq_token[j] : j] : -1;
        __syncthreads();
        // requests base + k before mine: longer ones, and equal ones with a smaller index
        const int before = i - base;  // k < before: a smaller index
#pragma unroll 8
        for (int k4 = 0; k4 < 256; k4 += 4) {
            const int4 o = *reinterpret_cast<const int4*>(&keys[k4]);
            rank += (o.x > mine || (o.x == mine && k4 + 0 < before)) ? 1 : 0;
            rank += (o.y > mine || (o.y == mine && k4 + 1 < before)) ? 1 : 0;
            rank += (o.z > mine || (o.z == mine && k4 + 2 < before)) ? 1 : 0;
            rank += (o.w > mine || (o.w == mine && k4 + 3 < before)) ? 1 : 0;
        }
    }
    if (i < n) order[rank] = i;
}

extern "C" int rl_order_by_length(const int* positions, const int* seq_token, int n, int* order,
                                  hipStream_t stream) {
    if (n <= 0) return RL_OK;
    if (!positions || !order) return RL_ERR_ARG;
    hipLaunchKernelGGL(order_by_length_kernel, dim3((n + 255) / 256), dim3(256), 0, stream,
                       positions, seq_token, n, order);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// A plain read of a buffer, for measuring what the memory system delivers: every thread
// keeps eight 16-byte loads in flight; nothing is written unless the data match a pattern
// that never occurs (so that the loads cannot be dropped).
// --------------------------------------------------------------------------- //
__global__ __launch_bounds__(256) void read_kernel(const uint4* __restrict__ src, size_t n16,
                                                   unsigned* __restrict__ sink) {
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t stride = (size_t)gridDim.x * blockDim.x;
    unsigned acc = 0;
    for (; i + 7 * stride < n16; i += 8 * stride) {
        uint4 v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = src[i + u * stride];
#pragma unroll
        for (int u = 0; u < 8; ++u) acc += v[u].x ^ v[u].y ^ v[u].z ^ v[u].w;
    }
    for (; i < n16; i += stride) acc += src[i].x;
    if (acc == 0x9e3779b9u) sink[0] = acc;
}

extern "C" int rl_read_buffer(const void* src, size_t bytes, unsigned* sink, int blocks,
                              hipStream_t stream) {
    if (bytes < 16 || blocks < 1 || (reinterpret_cast<uintptr_t>(src) & 15)) return RL_ERR_ARG;
    hipLaunchKernelGGL(read_kernel, dim3(blocks), dim3(256), 0, stream, (const uint4*)src,
                       bytes / 16, sink);
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// An activation over a token's whole hidden vector z (in place or not):
//   out = a N(z) + b N(z^2) + c N(z^3) + e,   N(y) = y / sqrt(mean(y^2) + eps),
// powers element by element, (a, b, c, e) = coef[0..3].  One workgroup a row; the three sums of
// squares and the result are float32, and a row's sums are formed in one order whatever the step.
// --------------------------------------------------------------------------- //
// three block-wide sums with one pair of barriers; `scratch` is a __shared__ float[48]
__device__ inline void block_sum3(float& a, float& b, float& c, float* scratch) {
    const int lane = threadIdx.x & (RL_WAVE - 1);
    const int wave = threadIdx.x / RL_WAVE;
    const int nwaves = (blockDim.x + RL_WAVE - 1) / RL_WAVE;
    a = wave_sum(a);
    b = wave_sum(b);
    c = wave_sum(c);
    __syncthreads();
    if (lane == 0) {
        scratch[wave] = a;
        scratch[16 + wave] = b;
        scratch[32 + wave] = c;
    }
    __syncthreads();
    a = b = c = 0.f;
    for (int i = 0; i < nwaves; ++i) {
        a += scratch[i];
        b += scratch[16 + i];
        c += scratch[32 + i];
    }
}

// VEC elements a thread and round (8 where the row allows 16-byte accesses, else 1)
template <typename T, int VEC>
__global__ __launch_bounds__(256) void polynorm_kernel(const T* __restrict__ x, T* __restrict__ out, int cols,
                                                       const float* __restrict__ coef, float eps) {
    struct alignas(sizeof(T) * VEC) Pack {
        T v[VEC];
    };
    __shared__ float scratch[48];
    const T* row = x + (size_t)blockIdx.x * cols;
    T* dst = out + (size_t)blockIdx.x * cols;
    float s2 = 0.f, s4 = 0.f, s6 = 0.f;
#pragma unroll 4
    for (int i = VEC * threadIdx.x; i < cols; i += VEC * blockDim.x) {
        const Pack in = *reinterpret_cast<const Pack*>(row + i);
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            const float z = to_float(in.v[e]);
            const float z2 = z * z;
            s2 += z2;
            s4 += z2 * z2;
            s6 += z2 * z2 * z2;
        }
    }
    block_sum3(s2, s4, s6, scratch);
    const float r1 = coef[0] * rsqrtf(s2 / (float)cols + eps);
    const float r2 = coef[1] * rsqrtf(s4 / (float)cols + eps);
    const float r3 = coef[2] * rsqrtf(s6 / (float)cols + eps);
    const float e0 = coef[3];
#pragma unroll 4
    for (int i = VEC * threadIdx.x; i < cols; i += VEC * blockDim.x) {
        const Pack in = *reinterpret_cast<const Pack*>(row + i);
        Pack o;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            const float z = to_float(in.v[e]);
            o.v[e] = from_float<T>(z * r1 + (z * z) * r2 + (z * z * z) * r3 + e0);
        }
        *reinterpret_cast<Pack*>(dst + i) = o;
    }
}

extern "C" int rl_polynorm(const void* x, void* out, int tokens, int cols, const float* coef, float eps,
                           int act_type, hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (cols < 1 || !coef) return RL_ERR_ARG;
    const bool vec = cols % 8 == 0;
    if (act_type == RL_F32 && vec)
        hipLaunchKernelGGL((polynorm_kernel<float, 8>), dim3(tokens), dim3(256), 0, stream, (const float*)x,
                           (float*)out, cols, coef, eps);
    else if (act_type == RL_F32)
        hipLaunchKernelGGL((polynorm_kernel<float, 1>), dim3(tokens), dim3(256), 0, stream, (const float*)x,
                           (float*)out, cols, coef, eps);
    else if (act_type == RL_BF16 && vec)
        hipLaunchKernelGGL((polynorm_kernel<bf16_t, 8>), dim3(tokens), dim3(256), 0, stream, (const bf16_t*)x,
                           (bf16_t*)out, cols, coef, eps);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL((polynorm_kernel<bf16_t, 1>), dim3(tokens), dim3(256), 0, stream, (const bf16_t*)x,
                           (bf16_t*)out, cols, coef, eps);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}

// --------------------------------------------------------------------------- //
// Finished logits in place (float32): v <- v * scale, then, with cap > 0, v <- cap * tanh(v / cap)
// --------------------------------------------------------------------------- //
__global__ void scale_cap_kernel(float* __restrict__ v, size_t total, float scale, float cap) {
    size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    const size_t step = (size_t)gridDim.x * blockDim.x;
    for (; idx < total; idx += step) {
        const float y = v[idx] * scale;
        v[idx] = cap > 0.f ? cap * tanhf(y / cap) : y;
    }
}

extern "C" int rl_scale_cap(float* v, size_t total, float scale, float cap, hipStream_t stream) {
    if (total == 0) return RL_OK;
    if (cap < 0.f) return RL_ERR_ARG;
    size_t blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    hipLaunchKernelGGL(scale_cap_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, v, total, scale, cap);
    return rl_launch_status();
}
