// Few-row GEMM for batched decode:  C[M,N] = epilogue( A[M,K] . W[N,K]^T ),  2 <= M <= 64, bf16.
//
// HBM-bound like the single-row GEMV (gemv.hip): every weight byte is read once, straight into MFMA A fragments. A workgroup owns
// 16 NT output columns; its NW waves take alternate 64-element slices of K (a row's slice is one whole 128-byte line), the batch rows
// are the columns of v_mfma_f32_16x16x32_bf16 (MT groups of 16), and the waves' partial tiles are summed through LDS in a fixed
// order.
#include "common.h"
#include "kernels.h"
#include "gemm_epilogue.h"
#include "debug.h"

namespace {

struct SkinnyArgs {
    const bf16_t* A; long lda;
    const bf16_t* W; long ldw;
    int M, N, K;
    EpiArgs epi;
};

template <int MT, int NT, int NW>
__global__ __launch_bounds__(64 * NW) void gemm_skinny_kernel(SkinnyArgs p) {
    constexpr int U = MT * NT <= 2 ? 4 : 2;         // 64-slices in flight per wave
    __shared__ __attribute__((aligned(16))) f32x4 red[NW][MT * NT][64];
    const int lane = threadIdx.x & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int n0 = blockIdx.x * (16 * NT);
    const bf16_t *w[NT], *a[MT];
    f32x4 acc[MT * NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) w[t] = p.W + (long)min(n0 + 16 * t + li, p.N - 1) * p.ldw + 8 * g;
#pragma unroll
    for (int t = 0; t < MT; ++t) a[t] = p.A + (long)min(16 * t + li, p.M - 1) * p.lda + 8 * g;
#pragma unroll
    for (int t = 0; t < MT * NT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int ns = p.K >> 6;
    for (int sl = wid; sl < ns; sl += NW * U) {
        u32x4 wf[U][NT][2], af[U][MT][2];
        // (slices past the end repeat the last one and are not multiplied: every load of a batch goes out at once)
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = 64 * min(sl + NW * u, ns - 1);
#pragma unroll
            for (int t = 0; t < NT; ++t)
#pragma unroll
                for (int hf = 0; hf < 2; ++hf) wf[u][t][hf] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(w[t] + k + 32 * hf));
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = 64 * min(sl + NW * u, ns - 1);
#pragma unroll
            for (int t = 0; t < MT; ++t)
#pragma unroll
                for (int hf = 0; hf < 2; ++hf) af[u][t][hf] = *reinterpret_cast<const u32x4*>(a[t] + k + 32 * hf);
        }
        __builtin_amdgcn_sched_barrier(0);          // (hipcc otherwise sinks the loads to their uses to save registers)
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (sl + NW * u >= ns) break;
#pragma unroll
            for (int t = 0; t < MT; ++t)
#pragma unroll
                for (int q = 0; q < NT; ++q)
#pragma unroll
                    for (int hf = 0; hf < 2; ++hf)
                        acc[t * NT + q] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf[u][q][hf]),
                                                                                  __builtin_bit_cast(bf16x8, af[u][t][hf]), acc[t * NT + q], 0, 0, 0);
        }
    }
#pragma unroll
    for (int t = 0; t < MT * NT; ++t) red[wid][t][lane] = acc[t];
    __syncthreads();
    if (wid >= MT * NT) return;
    f32x4 v = red[0][wid][lane];
#pragma unroll
    for (int s = 1; s < NW; ++s) v += red[s][wid][lane];
    const int m = 16 * (wid / NT) + li, n = n0 + 16 * (wid % NT) + 4 * g;
    if (m < p.M && n < p.N) epilogue4<bf16_t>(p.epi, m, n, v);
}

}  // namespace

bool cogs_k_gemm_skinny_fits(const CogsGemm& g) {
    return g.dtype == COGS_DT_BF16 && g.M >= 2 && g.M <= 64 && g.K % 64 == 0 && g.N % 4 == 0 && g.lda % 8 == 0 && g.ldw % 8 == 0 &&
           !g.rms_gamma && !g.row_stats && !g.ln_ab && !g.kv_k && g.hm_rows == 0;
}

int cogs_k_gemm_skinny(hipStream_t st, const CogsGemm& g) {
    if (!cogs_k_gemm_skinny_fits(g)) return COGS_E_UNSUPPORTED;
    SkinnyArgs p;
    const int rc = cogs_fill_epi(g, &p.epi);
    if (rc != COGS_OK) return rc;
    p.A = (const bf16_t*)g.A; p.lda = g.lda; p.W = (const bf16_t*)g.W; p.ldw = g.ldw;
    p.M = g.M; p.N = g.N; p.K = g.K;
    const bool deep = g.K >= 1024;
    const bool two = g.N >= 8192 && g.M <= 32;      // enough workgroups with 32 columns each: half the reads of A
    const int grid = two ? (g.N + 31) / 32 : (g.N + 15) / 16;
    g_cogs_debug.gemm_last_body = 7;
#define COGS_SKINNY(MT, NT)                                                                                       \
    do {                                                                                                          \
        if (deep) hipLaunchKernelGGL((gemm_skinny_kernel<MT, NT, 8>), dim3(grid), dim3(512), 0, st, p);            \
        else hipLaunchKernelGGL((gemm_skinny_kernel<MT, NT, 4>), dim3(grid), dim3(256), 0, st, p);                 \
    } while (0)
    if (g.M <= 16) { if (two) COGS_SKINNY(1, 2); else COGS_SKINNY(1, 1); }
    else if (g.M <= 32) { if (two) COGS_SKINNY(2, 2); else COGS_SKINNY(2, 1); }
    else COGS_SKINNY(4, 1);
#undef COGS_SKINNY
    return COGS_LAUNCH_CHECK();
}
