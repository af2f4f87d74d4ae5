// Small Qwen2-side helpers: KV-cache append, greedy argmax, HF logits processors, top-k.
//
// Replaces (third-party, transformers==4.46.3 as pinned by environment.yml:404):
//   DynamicCache.update (KV append), GenerationMixin greedy argmax,
//   RepetitionPenaltyLogitsProcessor / TemperatureLogitsWarper / TopKLogitsWarper
//   (model/generation_config.json:2-12) and the allowed-token mask of
//   StructuredLogitsProcessor (model/qaselect_module_predict.py:86-103).
#include "common.h"
#include "kernels.h"

namespace {

__global__ __launch_bounds__(256) void copy_cols_kernel(const char* __restrict__ src, long ld_src,
                                                        char* __restrict__ dst, long ld_dst, int rows, int chunks) {
    const long total = (long)rows * chunks;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
        const long r = i / chunks;
        const int c = (int)(i % chunks);
        *reinterpret_cast<u32x4*>(dst + r * ld_dst + c * 16) = *reinterpret_cast<const u32x4*>(src + r * ld_src + c * 16);
    }
}

__global__ __launch_bounds__(256) void kv_append_kernel(const char* __restrict__ ks, const char* __restrict__ vs,
                                                        long ld_src, char* __restrict__ kd, char* __restrict__ vd,
                                                        long ld_dst, int rows, int chunks) {
    const long total = (long)rows * chunks * 2;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
        const int which = (int)(i & 1);
        const long j = i >> 1;
        const long r = j / chunks;
        const int c = (int)(j % chunks);
        const char* s = (which ? vs : ks) + r * ld_src + c * 16;
        char* d = (which ? vd : kd) + r * ld_dst + c * 16;
        *reinterpret_cast<u32x4*>(d) = *reinterpret_cast<const u32x4*>(s);
    }
}

// first-maximum argmax, two stages
constexpr int AM_BLOCKS = 64;
__global__ __launch_bounds__(256) void argmax_part_kernel(const float* __restrict__ x, int n, float* __restrict__ ws) {
    __shared__ float sv[4];
    __shared__ int si[4];
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = blockIdx.x * 256 + threadIdx.x; i < n; i += AM_BLOCKS * 256) {
        const float v = x[i];
        if (v > bv || (v == bv && i < bi)) { bv = v; bi = i; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
        const float ov = __shfl_xor(bv, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    if (lane == 0) { sv[wid] = bv; si[wid] = bi; }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 4; ++w)
            if (sv[w] > bv || (sv[w] == bv && si[w] < bi)) { bv = sv[w]; bi = si[w]; }
        ws[blockIdx.x] = bv;
        reinterpret_cast<int*>(ws)[AM_BLOCKS + blockIdx.x] = bi;
    }
}
__global__ __launch_bounds__(64) void argmax_final_kernel(const float* __restrict__ ws, int64_t* __restrict__ out) {
    const int lane = threadIdx.x;
    float bv = ws[lane];
    int bi = reinterpret_cast<const int*>(ws)[AM_BLOCKS + lane];
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
        const float ov = __shfl_xor(bv, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    if (lane == 0) out[0] = bi == 0x7fffffff ? 0 : bi;
}

__global__ __launch_bounds__(1024) void logits_process_kernel(float* __restrict__ logits, int n,
                                                              const int64_t* __restrict__ prev, int n_prev, float pen,
                                                              const int32_t* __restrict__ allowed, int n_allowed,
                                                              float temperature, float* __restrict__ tmp) {
    const int tid = threadIdx.x;
    if (n_prev > 0 && pen != 1.0f) {
        for (int i = tid; i < n_prev; i += 1024) tmp[i] = logits[prev[i]];
        __syncthreads();
        for (int i = tid; i < n_prev; i += 1024) {
            const float s = tmp[i];
            logits[prev[i]] = s < 0.f ? s * pen : s / pen;
        }
        __syncthreads();
    }
    if (n_allowed > 0) {
        __shared__ float keep[256];
        for (int i = tid; i < n_allowed; i += 1024) keep[i] = logits[allowed[i]];
        __syncthreads();
        for (int i = tid; i < n; i += 1024) logits[i] = -INFINITY;
        __syncthreads();
        for (int i = tid; i < n_allowed; i += 1024) logits[allowed[i]] = keep[i];
        __syncthreads();
    }
    if (temperature != 1.0f)
        for (int i = tid; i < n; i += 1024) logits[i] = logits[i] / temperature;
}

__global__ __launch_bounds__(1024) void topk_kernel(const float* __restrict__ logits, int n, int k,
                                                    float* __restrict__ tv, int32_t* __restrict__ ti,
                                                    float* __restrict__ work) {
    __shared__ float sv[16];
    __shared__ int si[16];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    for (int i = tid; i < n; i += 1024) work[i] = logits[i];
    __syncthreads();
    for (int r = 0; r < k; ++r) {
        float bv = -INFINITY;
        int bi = 0x7fffffff;
        for (int i = tid; i < n; i += 1024) {
            const float v = work[i];
            if (v > bv || (v == bv && i < bi)) { bv = v; bi = i; }
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ov = __shfl_xor(bv, o, 64);
            const int oi = __shfl_xor(bi, o, 64);
            if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
        }
        if (lane == 0) { sv[wid] = bv; si[wid] = bi; }
        __syncthreads();
        if (tid == 0) {
            for (int w = 1; w < 16; ++w)
                if (sv[w] > bv || (sv[w] == bv && si[w] < bi)) { bv = sv[w]; bi = si[w]; }
            tv[r] = bv;
            ti[r] = bi == 0x7fffffff ? -1 : bi;
            if (bi != 0x7fffffff) work[bi] = -INFINITY;
            // a row of all -inf keeps returning -1; the host treats that as "fewer than k candidates"
        }
        __syncthreads();
    }
}

// sequence and position of every new row of a step
__global__ __launch_bounds__(256) void seq_rows_kernel(const CogsSeq* __restrict__ seqs, int nseq, int rows, int* __restrict__ rowseq,
                                                       int* __restrict__ rowpos) {
    const int r = blockIdx.x * 256 + threadIdx.x;
    if (r >= rows) return;
    int lo = 0, hi = nseq;
    while (hi - lo > 1) { const int mid = (lo + hi) >> 1; if (seqs[mid].row0 <= r) lo = mid; else hi = mid; }
    rowseq[r] = lo;
    rowpos[r] = seqs[lo].pos0 + r - seqs[lo].row0;
}

__global__ __launch_bounds__(256) void rope_sets_kernel(float* __restrict__ table, const CogsRopeSet* __restrict__ sets,
                                                        const int* __restrict__ rowpos, int rows) {
    const CogsRopeSet s = sets[blockIdx.y];
    const long total = (long)rows * s.pairs;
    f32x2* out = reinterpret_cast<f32x2*>(table + s.off * rows);
    for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < total; i += (long)gridDim.x * 256) {
        const int r = (int)(i / s.pairs), p = (int)(i % s.pairs) - s.first;
        f32x2 cs = {1.f, 0.f};
        if (p >= 0 && p < s.n) {
            // the angle reaches thousands of radians: whole turns are removed in fp64, the fp32 functions see |a| <= pi
            const double turns = (double)rowpos[r] * s.freq[p] * 0.15915494309189535;
            const float a = (float)((turns - rint(turns)) * 6.283185307179586);
            cs = f32x2{cosf(a) * s.mag, sinf(a) * s.mag};
        }
        out[i] = cs;
    }
}

__global__ __launch_bounds__(256) void zero_kernel(u32x4* __restrict__ p, long n) {
    for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long)gridDim.x * 256) p[i] = u32x4{0, 0, 0, 0};
}

}  // namespace

int cogs_k_seq_rows(hipStream_t st, const CogsSeq* seqs, int nseq, int rows, int* rowseq, int* rowpos) {
    if (nseq <= 0 || rows <= 0) return COGS_E_INVALID;
    hipLaunchKernelGGL(seq_rows_kernel, dim3((rows + 255) / 256), dim3(256), 0, st, seqs, nseq, rows, rowseq, rowpos);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_rope_sets(hipStream_t st, float* table, const CogsRopeSet* sets_dev, int nsets, int max_pairs, const int* rowpos, int rows) {
    if (nsets <= 0 || rows <= 0 || max_pairs <= 0) return COGS_E_INVALID;
    long g = ((long)rows * max_pairs + 255) / 256;
    if (g > 2048) g = 2048;
    hipLaunchKernelGGL(rope_sets_kernel, dim3((unsigned)g, nsets), dim3(256), 0, st, table, sets_dev, rowpos, rows);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_zero(hipStream_t st, void* p, size_t bytes) {
    if (!p || bytes % 16) return COGS_E_INVALID;
    if (!bytes) return COGS_OK;
    long g = ((long)(bytes / 16) + 255) / 256;
    if (g > 2048) g = 2048;
    hipLaunchKernelGGL(zero_kernel, dim3((unsigned)g), dim3(256), 0, st, (u32x4*)p, (long)(bytes / 16));
    return COGS_LAUNCH_CHECK();
}

int cogs_k_copy_cols(hipStream_t st, int dtype, const void* src, long ld_src, void* dst, long ld_dst, int rows, int cols) {
    if (rows <= 0 || cols <= 0) return COGS_OK;
    const int es = dtype == COGS_DT_BF16 ? 2 : 4;
    if ((cols * es) % 16 || (ld_src * es) % 16 || (ld_dst * es) % 16) return COGS_E_INVALID;
    const int chunks = cols * es / 16;
    long g = ((long)rows * chunks + 255) / 256;
    if (g > 2048) g = 2048;
    hipLaunchKernelGGL(copy_cols_kernel, dim3((unsigned)g), dim3(256), 0, st, (const char*)src, ld_src * es, (char*)dst,
                       ld_dst * es, rows, chunks);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_kv_append(hipStream_t st, int dtype, const void* k_src, const void* v_src, long ld_src, void* k_dst,
                     void* v_dst, long ld_dst, int rows, int cols) {
    if (rows <= 0 || cols <= 0) return COGS_OK;
    const int es = dtype == COGS_DT_BF16 ? 2 : 4;
    if ((cols * es) % 16 || (ld_src * es) % 16 || (ld_dst * es) % 16) return COGS_E_INVALID;
    const int chunks = cols * es / 16;
    long g = ((long)rows * chunks * 2 + 255) / 256;
    if (g > 2048) g = 2048;
    hipLaunchKernelGGL(kv_append_kernel, dim3((unsigned)g), dim3(256), 0, st, (const char*)k_src, (const char*)v_src,
                       ld_src * es, (char*)k_dst, (char*)v_dst, ld_dst * es, rows, chunks);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_argmax(hipStream_t st, const float* logits, int n, int64_t* out, float* ws) {
    if (n <= 0) return COGS_E_INVALID;
    hipLaunchKernelGGL(argmax_part_kernel, dim3(AM_BLOCKS), dim3(256), 0, st, logits, n, ws);
    hipLaunchKernelGGL(argmax_final_kernel, dim3(1), dim3(64), 0, st, ws, out);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_logits_process(hipStream_t st, float* logits, int n, const int64_t* prev, int n_prev, float rep_penalty,
                          const int32_t* allowed, int n_allowed, float temperature, float* tmp) {
    if (n <= 0 || n_allowed > 256) return COGS_E_INVALID;
    hipLaunchKernelGGL(logits_process_kernel, dim3(1), dim3(1024), 0, st, logits, n, prev, n_prev, rep_penalty, allowed,
                       n_allowed, temperature, tmp);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_topk(hipStream_t st, const float* logits, int n, int top_k, float* topk_val, int32_t* topk_idx, float* ws) {
    if (n <= 0 || top_k <= 0 || top_k > 1024) return COGS_E_INVALID;
    hipLaunchKernelGGL(topk_kernel, dim3(1), dim3(1024), 0, st, logits, n, top_k, topk_val, topk_idx, ws);
    return COGS_LAUNCH_CHECK();
}
