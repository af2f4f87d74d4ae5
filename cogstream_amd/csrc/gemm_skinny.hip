// Few-row GEMM for batched decode:  C[M,N] = epilogue( A[M,K] . W[N,K]^T ),  2 <= M <= 64, bf16.
//
// HBM-bound like the single-row GEMV (gemv.hip): every weight byte is read once, straight into MFMA A fragments. A workgroup owns
// 16 output columns; its NW waves take alternate 64-element slices of K (a row's slice is one whole 128-byte line), the batch rows
// are the columns of v_mfma_f32_16x16x32_bf16 (MT groups of 16), and the waves' partial tiles are summed through LDS in a fixed
// order. The K index a lane covers is permuted the same way in both operands: in a 64-slice, lane group g holds 16 g .. 16 g + 15.
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

template <int MT, int NW>
__global__ __launch_bounds__(64 * NW) void gemm_skinny_kernel(SkinnyArgs p) {
    constexpr int U = MT == 1 ? 4 : 2;              // 64-slices in flight per wave
    __shared__ __attribute__((aligned(16))) f32x4 red[NW][MT][64];
    const int lane = threadIdx.x & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int n0 = blockIdx.x * 16;
    const bf16_t* w = p.W + (long)min(n0 + li, p.N - 1) * p.ldw + 16 * g;
    const bf16_t* a[MT];
    f32x4 acc[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        a[t] = p.A + (long)min(16 * t + li, p.M - 1) * p.lda + 16 * g;
        acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int ns = p.K >> 6;
    auto mma = [&](const u32x4& wf, const u32x4& af, f32x4& c) {
        c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf), __builtin_bit_cast(bf16x8, af), c, 0, 0, 0);
    };
    int sl = wid;
    for (; sl + NW * (U - 1) < ns; sl += NW * U) {
        u32x4 wf[U][2], af[U][MT][2];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int hf = 0; hf < 2; ++hf)
                wf[u][hf] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(w + 64 * (sl + NW * u) + 8 * hf));
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int t = 0; t < MT; ++t)
#pragma unroll
                for (int hf = 0; hf < 2; ++hf) af[u][t][hf] = *reinterpret_cast<const u32x4*>(a[t] + 64 * (sl + NW * u) + 8 * hf);
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int t = 0; t < MT; ++t)
#pragma unroll
                for (int hf = 0; hf < 2; ++hf) mma(wf[u][hf], af[u][t][hf], acc[t]);
    }
    for (; sl < ns; sl += NW)
#pragma unroll
        for (int hf = 0; hf < 2; ++hf) {
            const u32x4 wf = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(w + 64 * sl + 8 * hf));
#pragma unroll
            for (int t = 0; t < MT; ++t) mma(wf, *reinterpret_cast<const u32x4*>(a[t] + 64 * sl + 8 * hf), acc[t]);
        }
#pragma unroll
    for (int t = 0; t < MT; ++t) red[wid][t][lane] = acc[t];
    __syncthreads();
    if (wid >= MT) return;
    f32x4 v = red[0][wid][lane];
#pragma unroll
    for (int s = 1; s < NW; ++s) v += red[s][wid][lane];
    const int m = 16 * wid + li, n = n0 + 4 * g;
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
    const int grid = (g.N + 15) / 16;
    const bool wide = g.K >= 1024;
    g_cogs_debug.gemm_last_body = 7;
#define COGS_SKINNY(MT)                                                                                       \
    do {                                                                                                      \
        if (wide) hipLaunchKernelGGL((gemm_skinny_kernel<MT, 8>), dim3(grid), dim3(512), 0, st, p);            \
        else hipLaunchKernelGGL((gemm_skinny_kernel<MT, 4>), dim3(grid), dim3(256), 0, st, p);                 \
    } while (0)
    if (g.M <= 16) COGS_SKINNY(1);
    else if (g.M <= 32) COGS_SKINNY(2);
    else COGS_SKINNY(4);
#undef COGS_SKINNY
    return COGS_LAUNCH_CHECK();
}
