// Head rows of softmax attention with per-head keys and values (cogs_attn_mixer) behind the fused projection (fp32): optional RMS norm of
// every query and key head row (no weight), the query's temperature, the score scale in log2 units, and the cache rows, padding
// included (a tile's rows past the end repeat a row's last columns under a weight of zero). The attention itself is mla.hip's.
#include "common.h"
#include "kernels.h"

namespace {

// a wave per head row (4 columns per lane and pass); gridDim.y workgroups share a row's heads
template <typename T, int E>
__global__ __launch_bounds__(256) void attn_heads_kernel(CogsAttnHeads p) {
    const int row = blockIdx.x, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int pos = p.rowpos[row];
    const CogsSeq s = p.seqs[p.rowseq[row]];
    float qs = p.scale * 1.4426950408889634f;
    if (p.temp_every > 0.0) qs *= 1.f + (float)p.temp_coef * logf((float)(floor((pos + 1) / p.temp_every) + 1.0));
    const float* t = p.t + (long)row * p.ldt;
    const int total = p.heads + 2 * p.kv_heads;
    for (int j = blockIdx.y * 4 + wid; j < total; j += 4 * gridDim.y) {
        const bool is_q = j < p.heads, is_k = !is_q && j < p.heads + p.kv_heads;
        const int kh = is_q ? 0 : (j - p.heads) % p.kv_heads, cols = is_q || is_k ? p.dkp : p.dvp, out_cols = is_q || is_k ? p.dkp : p.kvw - p.dkp;
        const float* x = t + (is_q || is_k ? (long)j * p.dkp : (long)(p.heads + p.kv_heads) * p.dkp + (long)kh * p.dvp);
        T* y = is_q ? reinterpret_cast<T*>(p.q) + (long)row * p.heads * p.dkp + (long)j * p.dkp
                    : reinterpret_cast<T*>(s.cache) + (p.layer_off + (long)kh * p.kvw) * s.max_len + (long)pos * p.kvw + (is_k ? 0 : p.dkp);
        f32x4 v[E];
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int d = 4 * lane + 256 * e;
            v[e] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (d < cols) v[e] = *reinterpret_cast<const f32x4*>(x + d);
#pragma unroll
            for (int i = 0; i < 4; ++i) ss += v[e][i] * v[e][i];
        }
        float f = is_q ? qs : 1.f;
        if (p.norm && (is_q || is_k)) f *= 1.f / sqrtf(wave_sum(ss) / (float)p.dim + p.eps);
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int d = 4 * lane + 256 * e;
            if (d < out_cols) st4_f<T>(y + d, v[e] * f);
        }
    }
}

template <typename T>
void launch(hipStream_t st, const CogsAttnHeads& a, int rows, int cols) {
    const dim3 grid(rows, rows <= 64 ? (a.heads + 2 * a.kv_heads + 3) / 4 : 1);       // few rows: latency
    if (cols <= 256) hipLaunchKernelGGL((attn_heads_kernel<T, 1>), grid, dim3(256), 0, st, a);
    else if (cols <= 512) hipLaunchKernelGGL((attn_heads_kernel<T, 2>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((attn_heads_kernel<T, 8>), grid, dim3(256), 0, st, a);
}

}  // namespace

int cogs_k_attn_heads(hipStream_t st, int dtype, const CogsAttnHeads& a, int rows) {
    if (rows <= 0) return COGS_OK;
    const int cols = a.dkp > a.kvw - a.dkp ? a.dkp : a.kvw - a.dkp;
    if (a.heads <= 0 || a.kv_heads <= 0 || a.dim <= 0 || a.dkp % 4 || a.dvp % 4 || a.ldt % 4 || a.kvw % 4 || a.dkp + a.dvp > a.kvw) return COGS_E_INVALID;
    if (cols > 2048) return COGS_E_UNSUPPORTED;
    if (dtype == COGS_DT_BF16) launch<bf16_t>(st, a, rows, cols);
    else launch<float>(st, a, rows, cols);
    return COGS_LAUNCH_CHECK();
}
