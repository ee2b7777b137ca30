// Paged causal attention, one workgroup per (token, query head), float32 arithmetic for
// any element type.  This is the whole attention of the float32 path and the fallback of
// the bfloat16 path for shapes the matrix-core kernels refuse.  It serves every token of a
// mixed batch alike: a token at absolute position pos of a request reads the keys
// [max(0, pos - window + 1), pos] of that request through its block table
// (window 0: all keys), which were written before this kernel runs.  With a window, the first
// keep_first keys of the request are read as well; a value head has dv channels, which need not
// be d; with `sink` the softmax's denominator has one more term, exp(0) or, with `sink_values`,
// exp of a number per query head: a key without a value.  With cap > 0 a scaled score s becomes
// cap * tanh(s / cap); with `slopes` (one number a query head) slope_h * (pos - j) is then taken
// off it; with `log_r1` and `log_r2` instead r1_h * ln(1 + r2_h * (pos - j)) is.  A token's heads lie
// side by side in a row of `out` of out_width elements; `out_scale` multiplies the finished outputs, and
// with `gate` the sigmoid of gate[t * gate_width + h * dv + c] channel c of head h.  With `chunked` a token
// sees the keys of its own chunk of `window` positions, counted from the request's first.
//
// Scores (q . k) / sqrt(d) (rapid_llm/modules/attention.py:62), online softmax over tiles
// of 256 keys in ascending order (rapid_llm/kernels/ops/attention/flashattention2_nopad.py:
// 138-168), query head h reads kv head h / (nq / nkv) (:85).  Masked keys contribute
// exactly zero (-inf scores, as in rapid_llm/kernels/ops/attention/flashdecoding.py:223-237).
#include "common.h"

#define ATT_THREADS 256

template <typename T>
__global__ __launch_bounds__(ATT_THREADS) void attention_generic_kernel(
    const T* __restrict__ q, const T* __restrict__ k_cache, const T* __restrict__ v_cache,
    T* __restrict__ out, const int* __restrict__ positions, const int* __restrict__ token_slot,
    const int* __restrict__ block_table, int table_stride, int page_size, int nq, int nkv, int d,
    int window, float scale, int dv, int keep_first, int sink, const float* __restrict__ sink_values,
    float cap, const float* __restrict__ slopes, const float* __restrict__ log_r1,
    const float* __restrict__ log_r2, int out_width, float out_scale, int chunked,
    const T* __restrict__ gate, int gate_width) {
    __shared__ float qs[256];
    __shared__ float ps[ATT_THREADS];
    __shared__ int key_page[ATT_THREADS];  // page * nkv + kv head of each key of the tile
    __shared__ int key_off[ATT_THREADS];
    __shared__ float scratch[16];

    const int t = blockIdx.x;
    const int h = blockIdx.y;
    const int hk = h / (nq / nkv);
    const int tid = threadIdx.x;
    const int pos = positions[t];
    const int* table = block_table + (size_t)token_slot[t] * table_stride;
    const int kend = pos + 1;
    const int kstart = window <= 0 ? 0 : (chunked ? pos / window * window : max(pos - window + 1, 0));
    // the keys read, in ascending order: the kept first ones below the window, then the window's
    const int kept = window > 0 ? min(keep_first, kstart) : 0;
    const int nkeys = kept + (kend - kstart);

    const T* qrow = q + ((size_t)t * nq + h) * d;
    if (tid < d) qs[tid] = to_float(qrow[tid]);
    __syncthreads();

    float m = -INFINITY, l = 0.f, acc = 0.f;
    for (int base = 0; base < nkeys; base += ATT_THREADS) {
        const int jl = base + tid;
        const int j = jl < kept ? jl : kstart + (jl - kept);
        float s = -INFINITY;
        if (jl < nkeys) {
            const int page = table[j / page_size];
            const int off = j % page_size;
            key_page[tid] = page * nkv + hk;
            key_off[tid] = off;
            const T* krow = k_cache + ((size_t)(page * nkv + hk) * page_size + off) * d;
            float dot = 0.f;
            for (int i = 0; i < d; ++i) dot = fmaf(qs[i], to_float(krow[i]), dot);
            s = dot * scale;
            if (cap > 0.f) s = cap * tanhf(s / cap);
            if (slopes) s -= slopes[h] * (float)(pos - j);
            if (log_r1) s -= log_r1[h] * logf(fmaf(log_r2[h], (float)(pos - j), 1.f));
        }
        const float tile_max = block_max(s, scratch);  // finite: the tile holds >= 1 key
        const float m_new = fmaxf(m, tile_max);
        const float p = (jl < nkeys) ? expf(s - m_new) : 0.f;
        ps[tid] = p;
        const float tile_sum = block_sum(p, scratch);  // syncs: ps, key_page, key_off visible
        const float alpha = expf(m - m_new);           // m = -inf on the first tile: 0
        l = l * alpha + tile_sum;
        m = m_new;
        if (tid < dv) {
            acc *= alpha;
            const int n = min(ATT_THREADS, nkeys - base);
            for (int jj = 0; jj < n; ++jj) {
                const T* vrow = v_cache + ((size_t)key_page[jj] * dv + tid) * page_size;
                acc = fmaf(ps[jj], to_float(vrow[key_off[jj]]), acc);
            }
        }
        __syncthreads();  // ps / key_* are rewritten by the next tile
    }
    if (sink) {
        // a key without a value: its score is 0, or a number of the head (never scaled); it may
        // lie above every real score, so the state is brought to the larger maximum first
        const float s0 = sink_values ? sink_values[h] : 0.f;
        const float m_new = fmaxf(m, s0);
        const float fa = expf(m - m_new);
        l = l * fa + expf(s0 - m_new);
        acc *= fa;
    }
    if (tid < dv) {
        float y = acc / l * out_scale;
        if (gate) y /= 1.f + expf(-to_float(gate[(size_t)t * gate_width + h * dv + tid]));
        out[(size_t)t * out_width + h * dv + tid] = from_float<T>(y);
    }
}

extern "C" int rl_attention_generic(const void* q, const void* k_cache, const void* v_cache,
                                    void* out, const int* positions, const int* token_slot,
                                    const int* block_table, int table_stride, int page_size,
                                    int tokens, int nq, int nkv, int d, int window, float scale,
                                    int dv, int keep_first, int sink, const float* sink_values, float cap,
                                    const float* slopes, const float* log_r1, const float* log_r2, int out_width,
                                    float out_scale, int chunked, const void* gate, int gate_width, int act_type,
                                    hipStream_t stream) {
    if (tokens <= 0) return RL_OK;
    if (cap < 0.f || !log_r1 != !log_r2 || out_width < nq * dv) return RL_ERR_ARG;
    if ((chunked && (window < 1 || keep_first)) || (gate && gate_width < nq * dv)) return RL_ERR_ARG;
    if (d < 1 || d > 256 || dv < 1 || dv > 256 || keep_first < 0 || nkv < 1 || nq % nkv || page_size < 1 ||
        nq > 65535)
        return RL_ERR_ARG;
    dim3 grid(tokens, nq), block(ATT_THREADS);
    if (act_type == RL_F32)
        hipLaunchKernelGGL(attention_generic_kernel<float>, grid, block, 0, stream,
                           (const float*)q, (const float*)k_cache, (const float*)v_cache,
                           (float*)out, positions, token_slot, block_table, table_stride,
                           page_size, nq, nkv, d, window, scale, dv, keep_first, sink, sink_values, cap, slopes,
                           log_r1, log_r2, out_width, out_scale, chunked, (const float*)gate, gate_width);
    else if (act_type == RL_BF16)
        hipLaunchKernelGGL(attention_generic_kernel<bf16_t>, grid, block, 0, stream,
                           (const bf16_t*)q, (const bf16_t*)k_cache, (const bf16_t*)v_cache,
                           (bf16_t*)out, positions, token_slot, block_table, table_stride,
                           page_size, nq, nkv, d, window, scale, dv, keep_first, sink, sink_values, cap, slopes,
                           log_r1, log_r2, out_width, out_scale, chunked, (const bf16_t*)gate, gate_width);
    else
        return RL_ERR_ARG;
    return rl_launch_status();
}
