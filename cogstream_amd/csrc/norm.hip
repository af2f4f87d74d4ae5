// Row normalisations: LayerNorm (ViT), RMSNorm (Qwen2), and post-LayerNorm fused with the
// 2x2 token merge.
//
// Replaces: nn.LayerNorm(1152, eps=1e-6) x(2*27+1) (model/modeling_videollama3_encoder.py:382-384,
// :475), post_layernorm + un-permute + F.interpolate(bilinear, 1/2) (:482-501; with the
// merge-window-major row order every 4 consecutive rows are one 2x2 window, so the bilinear
// half-size resample is their mean), and transformers' Qwen2RMSNorm (fp32 variance,
// x*rsqrt(var+eps) cast back, then * weight).
//
// HBM-bound: one wave per row, the row lives in registers (16-byte loads, 8 elements per
// lane per chunk), statistics by 64-lane butterfly, one read + one write per element.
#include "common.h"
#include "kernels.h"

namespace {

template <typename T, int CPL, bool RMS>
__global__ __launch_bounds__(256) void norm_kernel(const T* __restrict__ x, T* __restrict__ y,
                                                   const T* __restrict__ gamma, const T* __restrict__ beta,
                                                   int rows, int H, float eps) {
    const int lane = threadIdx.x & 63;
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= rows) return;
    const int nch = H >> 3;
    const T* xr = x + (long)row * H;
    float v[CPL][8];
    float sum = 0.f;
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int ch = lane + 64 * c;
        if (ch < nch) {
            ld8_f<T>(xr + ch * 8, v[c]);
#pragma unroll
            for (int e = 0; e < 8; ++e) sum += RMS ? v[c][e] * v[c][e] : v[c][e];
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) v[c][e] = 0.f;
        }
    }
    sum = wave_sum(sum);
    float mean = 0.f, rstd;
    if (RMS) {
        rstd = rsqrtf(sum / (float)H + eps);
    } else {
        mean = sum / (float)H;
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
            const int ch = lane + 64 * c;
            if (ch < nch) {
#pragma unroll
                for (int e = 0; e < 8; ++e) { const float d = v[c][e] - mean; sq += d * d; }
            }
        }
        sq = wave_sum(sq);
        rstd = rsqrtf(sq / (float)H + eps);
    }
    T* yr = y + (long)row * H;
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int ch = lane + 64 * c;
        if (ch < nch) {
            float gm[8], o[8];
            ld8_f<T>(gamma + ch * 8, gm);
            if (RMS) {
                // Qwen2RMSNorm: weight * (x*rstd).to(input_dtype)
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    float n = v[c][e] * rstd;
                    if (sizeof(T) == 2) n = bf2f(f2bf(n));
                    o[e] = gm[e] * n;
                }
            } else {
                float bt[8];
                ld8_f<T>(beta + ch * 8, bt);
#pragma unroll
                for (int e = 0; e < 8; ++e) o[e] = (v[c][e] - mean) * rstd * gm[e] + bt[e];
            }
            st8_f<T>(yr + ch * 8, o);
        }
    }
}

template <typename T, int CPL>
__global__ __launch_bounds__(256) void ln_merge_kernel(const T* __restrict__ x, T* __restrict__ y,
                                                       const T* __restrict__ gamma, const T* __restrict__ beta,
                                                       int out_rows, int group, int H, float eps) {
    const int lane = threadIdx.x & 63;
    const int orow = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (orow >= out_rows) return;
    const int nch = H >> 3;
    float acc[CPL][8];
#pragma unroll
    for (int c = 0; c < CPL; ++c)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[c][e] = 0.f;
    for (int gidx = 0; gidx < group; ++gidx) {
        const T* xr = x + ((long)orow * group + gidx) * H;
        float v[CPL][8];
        float sum = 0.f;
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
            const int ch = lane + 64 * c;
            if (ch < nch) {
                ld8_f<T>(xr + ch * 8, v[c]);
#pragma unroll
                for (int e = 0; e < 8; ++e) sum += v[c][e];
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) v[c][e] = 0.f;
            }
        }
        sum = wave_sum(sum);
        const float mean = sum / (float)H;
        float sq = 0.f;
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
            const int ch = lane + 64 * c;
            if (ch < nch) {
#pragma unroll
                for (int e = 0; e < 8; ++e) { const float d = v[c][e] - mean; sq += d * d; }
            }
        }
        sq = wave_sum(sq);
        const float rstd = rsqrtf(sq / (float)H + eps);
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
            const int ch = lane + 64 * c;
            if (ch < nch) {
                float gm[8], bt[8];
                ld8_f<T>(gamma + ch * 8, gm);
                ld8_f<T>(beta + ch * 8, bt);
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    float n = (v[c][e] - mean) * rstd * gm[e] + bt[e];
                    if (sizeof(T) == 2) n = bf2f(f2bf(n));  // post_layernorm output is stored in T
                    acc[c][e] += n;
                }
            }
        }
    }
    const float invg = 1.0f / (float)group;
    T* yr = y + (long)orow * H;
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int ch = lane + 64 * c;
        if (ch < nch) {
            float o[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = acc[c][e] * invg;
            st8_f<T>(yr + ch * 8, o);
        }
    }
}

template <typename T, bool RMS>
int launch_norm(hipStream_t st, const void* x, void* y, const void* g, const void* b, int rows, int H, float eps) {
    const int cpl = (H / 8 + 63) / 64;
    dim3 grid((rows + 3) / 4), blk(256);
#define COGS_NORM_CASE(C)                                                                             \
    hipLaunchKernelGGL((norm_kernel<T, C, RMS>), grid, blk, 0, st, (const T*)x, (T*)y, (const T*)g, \
                       (const T*)b, rows, H, eps)
    if (cpl <= 1) COGS_NORM_CASE(1);
    else if (cpl <= 2) COGS_NORM_CASE(2);
    else if (cpl <= 3) COGS_NORM_CASE(3);
    else if (cpl <= 4) COGS_NORM_CASE(4);
    else if (cpl <= 8) COGS_NORM_CASE(8);
    else return COGS_E_UNSUPPORTED;
#undef COGS_NORM_CASE
    return COGS_LAUNCH_CHECK();
}

template <typename T>
int launch_ln_merge(hipStream_t st, const void* x, void* y, const void* g, const void* b, int out_rows, int group,
                    int H, float eps) {
    const int cpl = (H / 8 + 63) / 64;
    dim3 grid((out_rows + 3) / 4), blk(256);
#define COGS_LNM_CASE(C)                                                                            \
    hipLaunchKernelGGL((ln_merge_kernel<T, C>), grid, blk, 0, st, (const T*)x, (T*)y, (const T*)g, \
                       (const T*)b, out_rows, group, H, eps)
    if (cpl <= 1) COGS_LNM_CASE(1);
    else if (cpl <= 2) COGS_LNM_CASE(2);
    else if (cpl <= 3) COGS_LNM_CASE(3);
    else if (cpl <= 4) COGS_LNM_CASE(4);
    else if (cpl <= 8) COGS_LNM_CASE(8);
    else return COGS_E_UNSUPPORTED;
#undef COGS_LNM_CASE
    return COGS_LAUNCH_CHECK();
}

// (a, b) = (rstd, -rstd * mean) of every row from the per-tile partial sums the producing GEMM's epilogue wrote
// (EPI_ROWSTAT): fixed-order fp64 combination, biased variance like nn.LayerNorm
__global__ __launch_bounds__(256) void ln_finalize_kernel(const float* __restrict__ part, int rows, int tiles, float inv_h,
                                                          float eps, float* __restrict__ ab) {
    const int r = blockIdx.x * 256 + threadIdx.x;
    if (r >= rows) return;
    const f32x2* p = reinterpret_cast<const f32x2*>(part) + (long)r * tiles;
    double s1 = 0.0, s2 = 0.0;
    for (int t = 0; t < tiles; ++t) { const f32x2 v = p[t]; s1 += (double)v[0]; s2 += (double)v[1]; }
    const double mean = s1 * inv_h;
    const double var = fmax(s2 * inv_h - mean * mean, 0.0);
    const float rstd = (float)(1.0 / sqrt(var + (double)eps));
    *reinterpret_cast<f32x2*>(ab + 2 * (long)r) = f32x2{rstd, (float)(-(double)rstd * mean)};
}

// fp32 residual stream around a sublayer (kernels.h, CogsStreamNorm): one workgroup of TPB threads per row, the row in
// registers (C chunks of four columns per thread). Norms entirely in fp32, one rounding of the normed row.
template <typename T, int C, int TPB>
__global__ __launch_bounds__(TPB) void stream_norm_kernel(CogsStreamNorm p) {
    constexpr int NW = TPB / 64;
    __shared__ float red[2][NW];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const long row = p.pick ? p.pick[blockIdx.x] : blockIdx.x;
    float* x = p.x + row * p.Hp;
    auto row_rstd = [&](float ss, int which) {
        ss = wave_sum(ss);
        if (lane == 0) red[which][wid] = ss;
        __syncthreads();
        ss = red[which][0];
#pragma unroll
        for (int w = 1; w < NW; ++w) ss += red[which][w];
        return 1.f / sqrtf(ss / (float)p.H + p.eps);
    };
    f32x4 v[C];
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int i = (tid + TPB * c) * 4;
        v[c] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i < p.Hp) v[c] = p.embeds ? ld4_f<T>(reinterpret_cast<const T*>(p.embeds) + row * p.Hp + i) : *reinterpret_cast<const f32x4*>(x + i);
    }
    if (p.y) {
        f32x4 y[C];
        float ss = 0.f;
#pragma unroll
        for (int c = 0; c < C; ++c) {
            const int i = (tid + TPB * c) * 4;
            y[c] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (i < p.Hp) y[c] = ld4_f<T>(reinterpret_cast<const T*>(p.y) + row * p.Hp + i);
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += y[c][e] * y[c][e];
        }
        if (p.y_gamma) {
            const float rs = row_rstd(ss, 0);
#pragma unroll
            for (int c = 0; c < C; ++c) {
                const int i = (tid + TPB * c) * 4;
                if (i >= p.Hp) continue;
                const f32x4 g = *reinterpret_cast<const f32x4*>(p.y_gamma + i);
#pragma unroll
                for (int e = 0; e < 4; ++e) y[c][e] = y[c][e] * rs * g[e];
            }
        }
#pragma unroll
        for (int c = 0; c < C; ++c) v[c] += y[c];
    }
    if (p.y || p.embeds) {
#pragma unroll
        for (int c = 0; c < C; ++c) {
            const int i = (tid + TPB * c) * 4;
            if (i < p.Hp) *reinterpret_cast<f32x4*>(x + i) = v[c];
        }
    }
    if (!p.out) return;
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += v[c][e] * v[c][e];
    const float rs = row_rstd(ss, 1);
    T* o = reinterpret_cast<T*>(p.out) + (long)blockIdx.x * p.Hp;
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int i = (tid + TPB * c) * 4;
        if (i >= p.Hp) continue;
        const f32x4 g = *reinterpret_cast<const f32x4*>(p.out_gamma + i);
        st4_f<T>(o + i, f32x4{v[c][0] * rs * g[0], v[c][1] * rs * g[1], v[c][2] * rs * g[2], v[c][3] * rs * g[3]});
    }
}

// the same with a scaled embedding and a position table at the start and hyper-connected streams (x [row][stream][Hp]). NS: streams
// rounded up; a chunk's old streams are in registers together, only the combination that is normed stays there for the row.
template <typename T, int C, int TPB, int NS>
__global__ __launch_bounds__(TPB) void stream_mix_kernel(CogsStreamNorm p) {
    constexpr int NW = TPB / 64;
    __shared__ float red[2][NW];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const long row = p.pick ? p.pick[blockIdx.x] : blockIdx.x;
    const int ns = p.streams > 0 ? p.streams : 1;
    float* x = p.x + row * ns * p.Hp;
    auto row_rstd = [&](float ss, int which) {
        ss = wave_sum(ss);
        if (lane == 0) red[which][wid] = ss;
        __syncthreads();
        ss = red[which][0];
#pragma unroll
        for (int w = 1; w < NW; ++w) ss += red[which][w];
        return 1.f / sqrtf(ss / (float)p.H + p.eps);
    };
    f32x4 y[C], u[C];
    float rs = 1.f;
    if (p.y) {
        float ss = 0.f;
#pragma unroll
        for (int c = 0; c < C; ++c) {
            const int i = (tid + TPB * c) * 4;
            y[c] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (i < p.Hp) y[c] = ld4_f<T>(reinterpret_cast<const T*>(p.y) + row * p.Hp + i);
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += y[c][e] * y[c][e];
        }
        if (p.y_gamma) rs = row_rstd(ss, 0);
    }
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int i = (tid + TPB * c) * 4;
        u[c] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i >= p.Hp) continue;
        f32x4 v[NS];
        if (p.embeds) {
            f32x4 e = ld4_f<T>(reinterpret_cast<const T*>(p.embeds) + row * p.Hp + i) * p.embed_scale;
            if (p.pos) e += ld4_f<T>(reinterpret_cast<const T*>(p.pos) + (long)p.rowpos[row] * p.Hp + i);
#pragma unroll
            for (int s = 0; s < NS; ++s) v[s] = e;
        } else {
#pragma unroll
            for (int s = 0; s < NS; ++s)
                if (s < ns) v[s] = *reinterpret_cast<const f32x4*>(x + (long)s * p.Hp + i);
        }
        if (p.y) {
            f32x4 yv = y[c];
            if (p.y_gamma) yv *= rs * *reinterpret_cast<const f32x4*>(p.y_gamma + i);
            if (p.mix) {
                f32x4 w[NS];
#pragma unroll
                for (int t = 0; t < NS; ++t) {
                    if (t >= ns) continue;
                    w[t] = yv * p.out_w[t];
#pragma unroll
                    for (int s = 0; s < NS; ++s)
                        if (s < ns) w[t] += v[s] * p.mix[s * ns + t];
                }
#pragma unroll
                for (int t = 0; t < NS; ++t)
                    if (t < ns) v[t] = w[t];
            } else {
                v[0] += yv;
            }
        }
        f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            if (s >= ns) continue;
            if (p.y || p.embeds) *reinterpret_cast<f32x4*>(x + (long)s * p.Hp + i) = v[s];
            sum += v[s];
            u[c] += p.in_w ? v[s] * p.in_w[s] : v[s];
        }
        if (p.sum) *reinterpret_cast<f32x4*>(p.sum + row * p.Hp + i) = sum;
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += u[c][e] * u[c][e];
    }
    if (!p.out) return;
    rs = row_rstd(ss, 1);
    T* o = reinterpret_cast<T*>(p.out) + (long)blockIdx.x * p.Hp;
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int i = (tid + TPB * c) * 4;
        if (i >= p.Hp) continue;
        st4_f<T>(o + i, u[c] * rs * *reinterpret_cast<const f32x4*>(p.out_gamma + i));
    }
}

template <typename T, int NS>
int launch_stream_mix(hipStream_t st, const CogsStreamNorm& a) {
    const dim3 grid(a.rows);
#define COGS_STREAM(C, TPB) hipLaunchKernelGGL((stream_mix_kernel<T, C, TPB, NS>), grid, dim3(TPB), 0, st, a)
    if (a.rows <= 64 && a.Hp > 1024) {
        if (a.Hp <= 4096) COGS_STREAM(1, 1024);
        else if (a.Hp <= 16384) COGS_STREAM(4, 1024);
        else return COGS_E_UNSUPPORTED;
    } else if (a.Hp <= 1024) COGS_STREAM(1, 256);
    else if (a.Hp <= 4096) COGS_STREAM(4, 256);
    else if (a.Hp <= 16384) COGS_STREAM(16, 256);
    else return COGS_E_UNSUPPORTED;
#undef COGS_STREAM
    return COGS_LAUNCH_CHECK();
}

template <typename T>
int launch_stream_norm(hipStream_t st, const CogsStreamNorm& a) {
    if (a.streams > 0 || a.pos || a.embed_scale != 1.f || a.sum) {
        if (a.streams <= 1) return launch_stream_mix<T, 1>(st, a);
        if (a.streams <= 2) return launch_stream_mix<T, 2>(st, a);
        if (a.streams <= 4) return launch_stream_mix<T, 4>(st, a);
        if (a.streams <= 8) return launch_stream_mix<T, 8>(st, a);
        if (a.streams <= 16) return launch_stream_mix<T, 16>(st, a);
        return COGS_E_UNSUPPORTED;
    }
    const dim3 grid(a.rows);
#define COGS_STREAM(C, TPB) hipLaunchKernelGGL((stream_norm_kernel<T, C, TPB>), grid, dim3(TPB), 0, st, a)
    if (a.rows <= 64 && a.Hp > 1024) {           // few rows: latency, not bandwidth -- more threads on each
        if (a.Hp <= 4096) COGS_STREAM(1, 1024);
        else if (a.Hp <= 8192) COGS_STREAM(2, 1024);
        else if (a.Hp <= 16384) COGS_STREAM(4, 1024);
        else return COGS_E_UNSUPPORTED;
    } else if (a.Hp <= 1024) COGS_STREAM(1, 256);
    else if (a.Hp <= 2048) COGS_STREAM(2, 256);
    else if (a.Hp <= 4096) COGS_STREAM(4, 256);
    else if (a.Hp <= 8192) COGS_STREAM(8, 256);
    else if (a.Hp <= 16384) COGS_STREAM(16, 256);
    else return COGS_E_UNSUPPORTED;
#undef COGS_STREAM
    return COGS_LAUNCH_CHECK();
}

}  // namespace

int cogs_k_stream_norm(hipStream_t st, int dtype, const CogsStreamNorm& a) {
    if (a.rows <= 0) return COGS_OK;
    if ((a.pos && !a.rowpos) || (a.y && a.streams > 0 && (!a.mix || !a.out_w)) || (a.streams <= 0 && (a.mix || a.in_w))) return COGS_E_INVALID;
    if (!a.x || a.Hp % 4 || a.H <= 0 || a.H > a.Hp || (a.out && !a.out_gamma) || (a.pick && (!a.out || a.y || a.embeds))) return COGS_E_INVALID;
    return dtype == COGS_DT_BF16 ? launch_stream_norm<bf16_t>(st, a) : launch_stream_norm<float>(st, a);
}

int cogs_k_layernorm(hipStream_t st, int dtype, const void* x, void* y, const void* gamma, const void* beta,
                     int rows, int H, float eps) {
    if (rows <= 0) return COGS_OK;
    if (H % 8) return COGS_E_INVALID;
    return dtype == COGS_DT_BF16 ? launch_norm<bf16_t, false>(st, x, y, gamma, beta, rows, H, eps)
                                 : launch_norm<float, false>(st, x, y, gamma, beta, rows, H, eps);
}

int cogs_k_rmsnorm(hipStream_t st, int dtype, const void* x, void* y, const void* gamma, int rows, int H, float eps) {
    if (rows <= 0) return COGS_OK;
    if (H % 8) return COGS_E_INVALID;
    return dtype == COGS_DT_BF16 ? launch_norm<bf16_t, true>(st, x, y, gamma, nullptr, rows, H, eps)
                                 : launch_norm<float, true>(st, x, y, gamma, nullptr, rows, H, eps);
}

int cogs_k_ln_merge(hipStream_t st, int dtype, const void* x, void* y, const void* gamma, const void* beta,
                    int out_rows, int group, int H, float eps) {
    if (out_rows <= 0) return COGS_OK;
    if (H % 8 || group <= 0) return COGS_E_INVALID;
    return dtype == COGS_DT_BF16 ? launch_ln_merge<bf16_t>(st, x, y, gamma, beta, out_rows, group, H, eps)
                                 : launch_ln_merge<float>(st, x, y, gamma, beta, out_rows, group, H, eps);
}

int cogs_k_ln_finalize(hipStream_t st, const float* stat_part, int rows, int tiles, int H, float eps, float* ab) {
    if (rows <= 0 || tiles <= 0 || H <= 0) return COGS_E_INVALID;
    hipLaunchKernelGGL(ln_finalize_kernel, dim3((rows + 255) / 256), dim3(256), 0, st, stat_part, rows, tiles, 1.0f / (float)H,
                       eps, ab);
    return COGS_LAUNCH_CHECK();
}
