// Multi-head latent attention (MLA): keys and values of all heads are linear images of ONE low-rank latent per token, so the
// cache holds a row [latent c | rotated key part shared by the heads] and nothing per head.
//
//   score(i, j, h) = q_h(i) . W_uk_h c(j) + qr_h(i) . kr(j)        value(j, h) = W_uv_h c(j)
//
// Two evaluations of the same sums:
//   prompt   W_uk c and W_uv c are EXPANDED for the whole context by one GEMM; attention then is ordinary multi-head attention
//            over head rows [W_uk_h c | kr] (mla_prefill_kernel: S^T = K.Q^T and O^T = V^T.P^T on MFMA, P in registers);
//   decode   W_uk is ABSORBED into the query, (W_uk_h^T q_h) . c, and W_uv is applied behind the sum over keys: every head of a
//            sequence reads the same cache row once (mla_decode_kernel: 16 heads are the 16 columns of an MFMA tile, the keys
//            are split over workgroups; mla_combine_kernel merges the splits).
// A row-wise kernel (any size, bf16 or fp32) serves the fp32 mode and sizes the MFMA kernels have no instance for.
//
// Scores are in log2 units everywhere (the query projection's epilogue multiplies by scale * log2 e before its rounding), so are
// the optional per-head sinks: a sink joins the softmax sum with no key and no value. The optional per-head output gate
// multiplies the finished head row.
//
// Padded sizes (zeros, by the packer): dn = unrotated query/key part, dr = rotated part (multiples of 8), dv = value
// (multiple of 16), a query head is [dn | dr | 0] in dq = 32-multiple columns; a cache row is [c: kvp = 64-multiple | kr:
// 32-multiple] = kvw columns.
#include "common.h"
#include "kernels.h"
#include "debug.h"

namespace {

__device__ __forceinline__ float col_max4(float x) {      // over the lanes {li, li+16, li+32, li+48}, result in all four
    const unsigned xb = __builtin_bit_cast(unsigned, x);
    const auto a = __builtin_amdgcn_permlane16_swap(xb, xb, false, false);
    const float y = fmaxf(__builtin_bit_cast(float, (unsigned)a[0]), __builtin_bit_cast(float, (unsigned)a[1]));
    const unsigned yb = __builtin_bit_cast(unsigned, y);
    const auto b = __builtin_amdgcn_permlane32_swap(yb, yb, false, false);
    return fmaxf(__builtin_bit_cast(float, (unsigned)b[0]), __builtin_bit_cast(float, (unsigned)b[1]));
}

// sums of up to two values over a 256-thread workgroup, result in every thread; `red` holds 8 floats
__device__ __forceinline__ void block_sum2(float& a, float& b, float* red) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    a = wave_sum(a);
    b = wave_sum(b);
    if (lane == 0) { red[wid] = a; red[4 + wid] = b; }
    __syncthreads();
    a = (red[0] + red[1]) + (red[2] + red[3]);
    b = (red[4] + red[5]) + (red[6] + red[7]);
    __syncthreads();
}

// ------------------------------------------------------------------------------------------------ latents
struct LatentArgs {
    const float* t; long ldt;            // fused down projection, fp32: [q latent | kv latent | key part | gate logits]
    int qr, qrp, kvr, kvp, dr, krc;      // true / padded query rank, true / padded kv rank, rotated key dims, cache columns of the key part
    int own_kv, gate_col, heads;         // gate_col < 0: no gate
    const float* q_norm; const float* kv_norm; float eps;
    const float* rope; int rope_pairs, rope_first;     // table [rows][rope_pairs][2]; the rotated part starts at pair rope_first
    void* cq; float* gate;
    const CogsSeq* seqs; const int* rowseq; const int* rowpos; long layer_off;
};

// one workgroup per new row: RMS norm of the query latent, RMS norm of the kv latent and rotation of the shared key part
// (both straight into the sequence's cache row), sigmoid of the gate logits
template <typename T>
__global__ __launch_bounds__(256) void mla_latent_kernel(LatentArgs p) {
    __shared__ float red[8];
    const int row = blockIdx.x, tid = threadIdx.x;
    const float* t = p.t + (long)row * p.ldt;
    float sq = 0.f, skv = 0.f;
    for (int i = tid * 4; i < p.qrp; i += 1024) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(t + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) sq += v[e] * v[e];
    }
    const float* tk = t + p.qrp;
    if (p.own_kv)
        for (int i = tid * 4; i < p.kvp; i += 1024) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(tk + i);
#pragma unroll
            for (int e = 0; e < 4; ++e) skv += v[e] * v[e];
        }
    block_sum2(sq, skv, red);
    const float rq = 1.f / sqrtf(sq / (float)p.qr + p.eps);
    T* cq = reinterpret_cast<T*>(p.cq) + (long)row * p.qrp;
    for (int i = tid * 4; i < p.qrp; i += 1024) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(t + i), g = *reinterpret_cast<const f32x4*>(p.q_norm + i);
        st4_f<T>(cq + i, f32x4{v[0] * rq * g[0], v[1] * rq * g[1], v[2] * rq * g[2], v[3] * rq * g[3]});
    }
    if (p.own_kv) {
        const CogsSeq s = p.seqs[p.rowseq[row]];
        const int kvw = p.kvp + p.krc;
        T* c = reinterpret_cast<T*>(s.cache) + p.layer_off * s.max_len + (long)p.rowpos[row] * kvw;
        const float rk = 1.f / sqrtf(skv / (float)p.kvr + p.eps);
        for (int i = tid * 4; i < p.kvp; i += 1024) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(tk + i), g = *reinterpret_cast<const f32x4*>(p.kv_norm + i);
            st4_f<T>(c + i, f32x4{v[0] * rk * g[0], v[1] * rk * g[1], v[2] * rk * g[2], v[3] * rk * g[3]});
        }
        const float* tr = tk + p.kvp;
        const float* cs = p.rope + ((long)row * p.rope_pairs + p.rope_first) * 2;
        for (int i = tid * 2; i < p.krc; i += 512) {
            float a = 0.f, b = 0.f;
            if (i < p.dr) {
                const float u = tr[i], v = tr[i + 1], co = cs[i], si = cs[i + 1];
                a = fmaf(-v, si, u * co);
                b = fmaf(u, si, v * co);
            }
            st_f<T>(c + p.kvp + i, a);
            st_f<T>(c + p.kvp + i + 1, b);
        }
    }
    if (p.gate_col >= 0)
        for (int i = tid; i < p.heads; i += 256) p.gate[(long)row * p.heads + i] = 1.f / (1.f + expf(-t[p.gate_col + i]));
}

// cached rows of every sequence of the batch, back to back (the expansion GEMM's A operand when there is more than one)
__global__ __launch_bounds__(256) void mla_gather_kernel(const CogsSeq* seqs, long layer_off, int row_bytes, int es, char* out) {
    const CogsSeq s = seqs[blockIdx.y];
    const int rows = s.pos0 + s.len;
    const long chunks = (long)rows * (row_bytes >> 4);
    const char* src = s.cache + layer_off * s.max_len * es;
    char* dst = out + (long)s.ctx0 * row_bytes;
    for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < chunks; i += (long)gridDim.x * 256)
        *reinterpret_cast<u32x4*>(dst + i * 16) = *reinterpret_cast<const u32x4*>(src + i * 16);
}

// ------------------------------------------------------------------------------------------------ per-head products
struct HeadGemmArgs {
    const void* X; long ldxb; int ldxh;     // x[b][h][k] at X + b * ldxb + h * ldxh + k
    const void* W;                          // [heads][N][K]
    void* Y; long ldyb; int ldyh;
    int B, heads, N, K;
    const float* gate;                      // [B][heads] or null
    int tail, tail_src, tail_n;             // y[N .. N+tail) = x[tail_src + j] for j < tail_n, else 0
};

// y[b][h][n] = sum_k x[b][h][k] W[h][n][k]: up to 16 batch rows are the MFMA columns, a wave owns 16 outputs of one head
__global__ __launch_bounds__(256) void head_gemm_bf16_kernel(HeadGemmArgs p) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, li = lane & 15, g = lane >> 4;
    const int h = blockIdx.y, b0 = blockIdx.z * 16, b = b0 + li;
    const int n0 = (blockIdx.x * 4 + wid) * 16;
    const bf16_t* x = reinterpret_cast<const bf16_t*>(p.X) + (long)min(b, p.B - 1) * p.ldxb + h * p.ldxh;
    bf16_t* y = reinterpret_cast<bf16_t*>(p.Y) + (long)min(b, p.B - 1) * p.ldyb + h * p.ldyh;
    if (n0 >= p.N) {
        if (n0 < p.N + p.tail && b < p.B) {
            const int j0 = n0 - p.N + 4 * g;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (j0 + e < p.tail) y[p.N + j0 + e] = j0 + e < p.tail_n ? x[p.tail_src + j0 + e] : (bf16_t)0;
        }
        return;
    }
    const bf16_t* w = reinterpret_cast<const bf16_t*>(p.W) + ((long)h * p.N + n0 + li) * p.K;
    f32x4 a0 = {0.f, 0.f, 0.f, 0.f}, a1 = a0;
    int k = 8 * g;
    for (; k + 96 < p.K; k += 128) {          // four 32-wide steps in flight
        u32x4 wf[4], xf[4];
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            wf[s] = *reinterpret_cast<const u32x4*>(w + k + 32 * s);
            xf[s] = *reinterpret_cast<const u32x4*>(x + k + 32 * s);
        }
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            f32x4& a = (s & 1) ? a1 : a0;
            a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf[s]), __builtin_bit_cast(bf16x8, xf[s]), a, 0, 0, 0);
        }
    }
    for (; k < p.K; k += 32) {
        const u32x4 wf = *reinterpret_cast<const u32x4*>(w + k), xf = *reinterpret_cast<const u32x4*>(x + k);
        a0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf), __builtin_bit_cast(bf16x8, xf), a0, 0, 0, 0);
    }
    a0 += a1;
    if (b < p.B) {
        if (p.gate) a0 *= p.gate[(long)b * p.heads + h];
        st4_f<bf16_t>(y + n0 + 4 * g, a0);
    }
}

// the same in fp32: one wave per (output, head, batch row)
__global__ __launch_bounds__(256) void head_gemm_f32_kernel(HeadGemmArgs p) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int h = blockIdx.y, b = blockIdx.z, n = blockIdx.x * 4 + wid;
    if (n >= p.N + p.tail) return;
    const float* x = reinterpret_cast<const float*>(p.X) + (long)b * p.ldxb + h * p.ldxh;
    float* y = reinterpret_cast<float*>(p.Y) + (long)b * p.ldyb + h * p.ldyh;
    if (n >= p.N) {
        if (lane == 0) y[n] = n - p.N < p.tail_n ? x[p.tail_src + n - p.N] : 0.f;
        return;
    }
    const float* w = reinterpret_cast<const float*>(p.W) + ((long)h * p.N + n) * p.K;
    float a = 0.f;
    for (int k = lane; k < p.K; k += 64) a = fmaf(w[k], x[k], a);
    a = wave_sum(a);
    if (p.gate) a *= p.gate[(long)b * p.heads + h];
    if (lane == 0) y[n] = a;
}

// ------------------------------------------------------------------------------------------------ row-wise attention
// One wave per (new row, head), two passes over the keys, fp32 arithmetic. absorbed: K, KR and V are the cache rows of the
// row's sequence (head stride 0), else the expanded buffers at the sequence's context rows.
constexpr int RW_DIM = 2304;             // query dims held in LDS
constexpr int RW_VREG = 32;              // value columns per lane: dv <= 2048
template <typename T>
__global__ __launch_bounds__(64) void mla_rowwise_kernel(CogsMla p) {
    __shared__ __attribute__((aligned(16))) float qs[RW_DIM];
    const int lane = threadIdx.x, row = blockIdx.x, h = blockIdx.y;
    const CogsSeq s = p.seqs[p.rowseq[row]];
    const int nkeys = s.pos0 + (row - s.row0) + 1;
    const T* q = reinterpret_cast<const T*>(p.Q) + (long)row * p.ldq + (long)h * p.q_head;
    for (int d = lane; d < p.dn + p.dr; d += 64) qs[d] = ld_f<T>(q + d);
    __syncthreads();
    const T *K, *KR, *V;
    if (p.absorbed) {
        K = V = reinterpret_cast<const T*>(s.cache) + p.layer_off * s.max_len;
        KR = K + p.kr_col;
    } else {
        K = reinterpret_cast<const T*>(p.K) + (long)s.ctx0 * p.ldk + (long)h * p.k_head;
        V = reinterpret_cast<const T*>(p.V) + (long)s.ctx0 * p.ldv + (long)h * p.v_head;
        KR = reinterpret_cast<const T*>(p.KR) + (long)s.ctx0 * p.ldkr;
    }
    auto score = [&](int j) {
        const T* k = K + (long)j * p.ldk;
        const T* kr = KR + (long)j * p.ldkr;
        f32x4 a = {0.f, 0.f, 0.f, 0.f};
        for (int d = 0; d < p.dn; d += 4) {
            const f32x4 kv = ld4_f<T>(k + d), qv = *reinterpret_cast<const f32x4*>(qs + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) a[e] = fmaf(kv[e], qv[e], a[e]);
        }
        for (int d = 0; d < p.dr; d += 4) {
            const f32x4 kv = ld4_f<T>(kr + d), qv = *reinterpret_cast<const f32x4*>(qs + p.dn + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) a[e] = fmaf(kv[e], qv[e], a[e]);
        }
        return (a[0] + a[1]) + (a[2] + a[3]);
    };
    float m = -INFINITY, l = 0.f;
    for (int j = lane; j < nkeys; j += 64) {
        const float sc = score(j), mn = fmaxf(m, sc);
        l = l * exp2f(m - mn) + exp2f(sc - mn);
        m = mn;
    }
    float M = wave_max(m);
    const float sink = p.sink ? p.sink[h] : -INFINITY;
    M = fmaxf(M, sink);
    l = (m == -INFINITY) ? 0.f : l * exp2f(m - M);
    float L = wave_sum(l);
    if (p.sink) L += exp2f(sink - M);
    const float inv = 1.f / L;
    float o[RW_VREG];
#pragma unroll
    for (int e = 0; e < RW_VREG; ++e) o[e] = 0.f;
    for (int j0 = 0; j0 < nkeys; j0 += 64) {
        const int j = j0 + lane;
        const float pj = j < nkeys ? exp2f(score(j) - M) * inv : 0.f;
        const int cnt = min(64, nkeys - j0);
        for (int jj = 0; jj < cnt; ++jj) {
            const float w = __shfl(pj, jj, 64);
            const T* v = V + (long)(j0 + jj) * p.ldv;
#pragma unroll
            for (int e = 0; e < RW_VREG; ++e) {
                const int d = lane + 64 * e;
                if (d < p.dv) o[e] = fmaf(w, ld_f<T>(v + d), o[e]);
            }
        }
    }
    const float gt = p.gate ? p.gate[(long)row * p.heads + h] : 1.f;
    T* O = reinterpret_cast<T*>(p.O) + (long)row * p.ldo + (long)h * p.o_head;
#pragma unroll
    for (int e = 0; e < RW_VREG; ++e) {
        const int d = lane + 64 * e;
        if (d < p.dv) st_f<T>(O + d, o[e] * gt);
    }
}

// ------------------------------------------------------------------------------------------------ prompt attention (bf16)
// 4 waves x 16 NQ query rows of one (sequence, head); 64-key tiles, register-staged (the next tile's loads are in flight during
// the compute), scores transposed so that a lane's S^T registers of key blocks 2c, 2c+1 are the B operand of the c-th 32-key step
// of O^T = V^T.P^T (see attn_decode.hip). The softmax sum is one more MFMA per step with an all-ones A operand, i.e. the sum of
// the bf16 weights that multiply V.
template <int KS, int DT, int NQ>
__global__ __launch_bounds__(256, 2) void mla_prefill_kernel(CogsMla p, int nqt) {
    constexpr int CHK = KS * 4;                  // 16-byte chunks of a K row in LDS
    constexpr int KRS = KS * 64;                 // K row stride, a multiple of 128 bytes (KS even)
    constexpr int VRS = DT * 32 + 32;            // V row stride, an odd multiple of 32 bytes (DT even)
    constexpr int PK = KS, PV = DT / 2;          // staged chunks per thread
    static_assert(KS % 2 == 0 && DT % 2 == 0, "row strides");
    extern __shared__ __attribute__((aligned(16))) char smem[];
    char* const Ks = smem;
    char* const Vs = smem + 64 * KRS;

    const int tid = threadIdx.x, lane = tid & 63;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, g = lane >> 4;
    // contiguous runs of (sequence, head) pairs per XCD: the query tiles of a head meet in one L2; long tiles first
    const int total = gridDim.x;
    int bid = blockIdx.x;
    {
        const int xcd = bid & 7, q = total >> 3, r = total & 7;
        bid = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (bid >> 3);
    }
    const int pair = bid / nqt, qt = nqt - 1 - bid % nqt;
    const int h = pair % p.heads;
    const CogsSeq s = p.seqs[pair / p.heads];
    const int q0 = qt * (64 * NQ);
    if (q0 >= s.len) return;

    const bf16_t* Q = reinterpret_cast<const bf16_t*>(p.Q) + (long)s.row0 * p.ldq + (long)h * p.q_head;
    const bf16_t* K = reinterpret_cast<const bf16_t*>(p.K) + (long)s.ctx0 * p.ldk + (long)h * p.k_head;
    const bf16_t* KR = reinterpret_cast<const bf16_t*>(p.KR) + (long)s.ctx0 * p.ldkr;
    const bf16_t* V = reinterpret_cast<const bf16_t*>(p.V) + (long)s.ctx0 * p.ldv + (long)h * p.v_head;
    const int ks = (p.dn + p.dr + 31) >> 5, dt = p.dv >> 4;
    const int nkc = p.dn >> 3, nc = (p.dn + p.dr) >> 3, nvc = p.dv >> 3;

    bf16x8 qf[NQ][KS];
    int qpos[NQ], qrow[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        qrow[i] = q0 + wid * 16 * NQ + 16 * i + li;
        const int rc = min(qrow[i], s.len - 1);
        qpos[i] = s.pos0 + rc;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            u32x4 v = {0, 0, 0, 0};
            if (k < ks) v = *reinterpret_cast<const u32x4*>(Q + (long)rc * p.ldq + 32 * k + 8 * g);
            qf[i][k] = __builtin_bit_cast(bf16x8, v);
        }
    }
    const int wave_hi = s.pos0 + min(q0 + wid * 16 * NQ + 16 * NQ, s.len) - 1;     // last position of the wave's rows
    const int wave_lo = s.pos0 + min(q0 + wid * 16 * NQ, s.len - 1);
    const int kend = s.pos0 + min(q0 + 64 * NQ, s.len);                             // keys the workgroup needs
    const int nt = (kend + 63) >> 6;

    f32x4 oacc[NQ][DT], lacc[NQ];
    float m[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        m[i] = -INFINITY;
        lacc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < DT; ++d) oacc[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const u32x4 ones_w = {0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u};
    const bf16x8 ones = __builtin_bit_cast(bf16x8, ones_w);

    u32x4 kreg[PK], vreg[PV];
    auto load_tile = [&](int t) {
        const int kb = t * 64, last = kend - 1;
#pragma unroll
        for (int i = 0; i < PK; ++i) {
            const int id = tid + 256 * i, r = id / CHK, c = id % CHK;
            const long j = min(kb + r, last);              // rows past the end repeat the last one; their scores are masked
            kreg[i] = u32x4{0, 0, 0, 0};
            if (c < nkc) kreg[i] = *reinterpret_cast<const u32x4*>(K + j * p.ldk + c * 8);
            else if (c < nc) kreg[i] = *reinterpret_cast<const u32x4*>(KR + j * p.ldkr + (c - nkc) * 8);
        }
#pragma unroll
        for (int i = 0; i < PV; ++i) {
            const int id = tid + 256 * i, r = id / (2 * DT), c = id % (2 * DT);
            const long j = min(kb + r, last);
            if (c < nvc) vreg[i] = *reinterpret_cast<const u32x4*>(V + j * p.ldv + c * 8);
        }
    };
    const int v_rd = (4 * g + (li >> 2)) * VRS + (li & 3) * 8;

    load_tile(0);
    for (int t = 0; t < nt; ++t) {
        __syncthreads();                       // the previous tile's fragment reads are done
#pragma unroll
        for (int i = 0; i < PK; ++i) {
            const int id = tid + 256 * i, r = id / CHK, c = id % CHK;
            *reinterpret_cast<u32x4*>(Ks + r * KRS + ((c ^ (r & 7)) << 4)) = kreg[i];
        }
#pragma unroll
        for (int i = 0; i < PV; ++i) {
            const int id = tid + 256 * i, r = id / (2 * DT), c = id % (2 * DT);
            if (c < nvc) *reinterpret_cast<u32x4*>(Vs + r * VRS + c * 16) = vreg[i];
        }
        __syncthreads();
        if (t + 1 < nt) load_tile(t + 1);
        const int kb = t * 64;
        if (kb > wave_hi) continue;            // (uniform per wave; every wave still meets the barriers above)

        f32x4 sacc[NQ][4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
#pragma unroll
            for (int i = 0; i < NQ; ++i) sacc[i][u] = f32x4{0.f, 0.f, 0.f, 0.f};
            const char* kr = Ks + (16 * u + li) * KRS;
#pragma unroll
            for (int k = 0; k < KS; ++k) {
                if (k >= ks) break;
                const bf16x8 kf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(kr + (((4 * k + g) ^ (li & 7)) << 4)));
#pragma unroll
                for (int i = 0; i < NQ; ++i) sacc[i][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i][k], sacc[i][u], 0, 0, 0);
            }
        }
        if (kb + 63 > wave_lo) {               // the diagonal (or the ragged end) crosses this tile
#pragma unroll
            for (int i = 0; i < NQ; ++i)
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (kb + 16 * u + 4 * g + r > qpos[i]) sacc[i][u][r] = -INFINITY;
        }
        bf16x8 pf[NQ][2];
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            float tm = -INFINITY;
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) tm = fmaxf(tm, sacc[i][u][r]);
            tm = col_max4(tm);
            const float mn = fmaxf(m[i], tm);                   // finite from the first tile on: key 0 is visible to every row
            if (__builtin_amdgcn_ballot_w64(mn > m[i]) != 0) {
                const float al = __builtin_amdgcn_exp2f(m[i] - mn);     // exp2(-inf) = 0 on the first tile
                lacc[i] *= al;
#pragma unroll
                for (int d = 0; d < DT; ++d) oacc[i][d] *= al;
                m[i] = mn;
            }
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                u32x4 w;
#pragma unroll
                for (int e2 = 0; e2 < 4; ++e2) {
                    const int e = 2 * e2;
                    w[e2] = pack_bf2(__builtin_amdgcn_exp2f(sacc[i][2 * c + (e >> 2)][e & 3] - m[i]),
                                     __builtin_amdgcn_exp2f(sacc[i][2 * c + ((e + 1) >> 2)][(e + 1) & 3] - m[i]));
                }
                pf[i][c] = __builtin_bit_cast(bf16x8, w);
            }
        }
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
            for (int i = 0; i < NQ; ++i) lacc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[i][c], lacc[i], 0, 0, 0);
#pragma unroll
        for (int d = 0; d < DT; ++d) {
            if (d >= dt) break;
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                const char* va = Vs + v_rd + 32 * c * VRS + 32 * d;
                const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va));
                const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va + 16 * VRS));
                const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
                const bf16x8 vf = __builtin_bit_cast(bf16x8, u32x4{l2[0], l2[1], h2[0], h2[1]});
#pragma unroll
                for (int i = 0; i < NQ; ++i) oacc[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[i][c], oacc[i][d], 0, 0, 0);
            }
        }
    }
    const float sink = p.sink ? p.sink[h] : -INFINITY;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        if (qrow[i] >= s.len) continue;
        float f;
        if (p.sink) {
            const float M = fmaxf(m[i], sink), a = exp2f(m[i] - M);
            f = a / (lacc[i][0] * a + exp2f(sink - M));
        } else f = 1.f / lacc[i][0];
        const long row = s.row0 + qrow[i];
        if (p.gate) f *= p.gate[row * p.heads + h];
        bf16_t* O = reinterpret_cast<bf16_t*>(p.O) + row * p.ldo + (long)h * p.o_head + 4 * g;
#pragma unroll
        for (int d = 0; d < DT; ++d)
            if (d < dt) st4_f<bf16_t>(O + 16 * d, oacc[i][d] * f);
    }
}

// ------------------------------------------------------------------------------------------------ decode attention (bf16)
// One new row per sequence. Workgroup = (split of the keys, 16 heads, sequence). A tile of TK cache rows is one contiguous run in
// memory; it goes through registers into LDS and is read twice there: as K rows (A operand of S^T = C.Q^T, wave w owns key block
// w) and transposed as V (A operand of O^T = C^T.P^T, wave w owns the latent columns 16 (w + 4 i)). The weights travel between
// the waves through LDS.
struct MlaDecodeArgs {
    const bf16_t* Q; long ldq; int q_head;
    const CogsSeq* seqs; long layer_off;
    int kvw, kvp, heads, nht, nsplit;
    float* part_o; float* part_ml;          // [seq][split][head][kvp] relative to part_ml[..][0]; [..][2] = (max, sum)
};

template <int TK, int DTW, int PER>
__global__ __launch_bounds__(256) void mla_decode_kernel(MlaDecodeArgs p) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    constexpr int PRS = TK * 2 + 16;
    const int RS = p.kvw * 2 + 32;                               // an odd multiple of 32 bytes (kvw % 32 == 0)
    char* const Ks = smem;
    char* const Qs = Ks + TK * RS;
    char* const Ps = Qs + 16 * RS;
    float* const cmax = reinterpret_cast<float*>(Ps + 16 * PRS);   // [4][16]

    const int tid = threadIdx.x, lane = tid & 63;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, g = lane >> 4;
    // the head tiles of a split sit 8 apart in the launch order = on one XCD: its L2 serves the second and later readers
    const int bid = blockIdx.x, slot = bid & 7, rest = bid >> 3;
    const int ht = rest % p.nht, split = (rest / p.nht) * 8 + slot;
    if (split >= p.nsplit) return;
    const int b = blockIdx.y, h0 = ht * 16;
    const CogsSeq s = p.seqs[b];
    const int kend = s.pos0 + 1;
    const unsigned nt_all = (unsigned)(kend + TK - 1) / TK;
    const int t_begin = (int)(nt_all * (unsigned)split / (unsigned)p.nsplit);
    const int t_end = (int)(nt_all * (unsigned)(split + 1) / (unsigned)p.nsplit);
    const long slot0 = ((long)b * p.nsplit + split) * p.heads;
    if (t_begin >= t_end) {                                        // nothing to do: an empty partial
        if (tid < 16 && h0 + tid < p.heads) { p.part_ml[(slot0 + h0 + tid) * 2] = -INFINITY; p.part_ml[(slot0 + h0 + tid) * 2 + 1] = 0.f; }
        return;
    }
    const char* cache = s.cache + p.layer_off * s.max_len * 2;
    const int row_bytes = p.kvw * 2, nch = p.kvw >> 3;             // 16-byte chunks of a row
    const int tile_chunks = TK * nch;
    const int dr_row = 256 / nch, dr_c = 256 % nch;

    u32x4 reg[PER];
    auto load_tile = [&](int t) {
        const char* base = cache + (long)t * TK * row_bytes;
        const int lim = min(TK, kend - t * TK) * nch - 1;           // chunks past the end repeat the last one (masked)
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int id = tid + 256 * i;
            if (256 * i < tile_chunks) reg[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(base + (long)min(id, lim) * 16));
        }
    };
    load_tile(t_begin);
    for (int id = tid; id < 16 * nch; id += 256) {
        const int r = id / nch, c = id - r * nch;
        u32x4 v = {0, 0, 0, 0};
        if (h0 + r < p.heads) v = *reinterpret_cast<const u32x4*>(p.Q + (long)b * p.ldq + (long)(h0 + r) * p.q_head + c * 8);
        *reinterpret_cast<u32x4*>(Qs + r * RS + c * 16) = v;
    }
    const int row_t = tid / nch, c_t = tid - row_t * nch;
    const int ks = p.kvw >> 5, dts = p.kvp >> 4;
    f32x4 oacc[DTW], lacc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int d = 0; d < DTW; ++d) oacc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY;
    const u32x4 ones_w = {0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u};
    const bf16x8 ones = __builtin_bit_cast(bf16x8, ones_w);
    const char* const qrd = Qs + li * RS + 16 * g;
    const char* const krd = Ks + (16 * wid + li) * RS + 16 * g;
    const char* const vrd = Ks + (4 * g + (li >> 2)) * RS + (li & 3) * 8;

    for (int t = t_begin; t < t_end; ++t) {
        if (t != t_begin) __syncthreads();                        // the previous tile's transposed reads are done
        {
            int r = row_t, c = c_t;
#pragma unroll
            for (int i = 0; i < PER; ++i) {
                if (tid + 256 * i < tile_chunks) *reinterpret_cast<u32x4*>(Ks + r * RS + c * 16) = reg[i];
                r += dr_row; c += dr_c;
                if (c >= nch) { c -= nch; ++r; }
            }
        }
        __syncthreads();
        if (t + 1 < t_end) load_tile(t + 1);
        const int nvalid = min(TK, kend - t * TK);
        f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = sa;
        if (16 * wid < TK) {
            int k = 0;
            for (; k + 1 < ks; k += 2) {
                const u32x4 k0 = *reinterpret_cast<const u32x4*>(krd + 64 * k), q0 = *reinterpret_cast<const u32x4*>(qrd + 64 * k);
                const u32x4 k1 = *reinterpret_cast<const u32x4*>(krd + 64 * k + 64), q1 = *reinterpret_cast<const u32x4*>(qrd + 64 * k + 64);
                sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, k0), __builtin_bit_cast(bf16x8, q0), sa, 0, 0, 0);
                sb = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, k1), __builtin_bit_cast(bf16x8, q1), sb, 0, 0, 0);
            }
            if (k < ks) {
                const u32x4 k0 = *reinterpret_cast<const u32x4*>(krd + 64 * k), q0 = *reinterpret_cast<const u32x4*>(qrd + 64 * k);
                sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, k0), __builtin_bit_cast(bf16x8, q0), sa, 0, 0, 0);
            }
            sa += sb;
            float tm = -INFINITY;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (16 * wid + 4 * g + r >= nvalid) sa[r] = -INFINITY;
                tm = fmaxf(tm, sa[r]);
            }
            tm = col_max4(tm);
            if (g == 0) cmax[wid * 16 + li] = tm;
        }
        __syncthreads();
        float mn = fmaxf(m, fmaxf(cmax[li], cmax[16 + li]));
        if constexpr (TK == 64) mn = fmaxf(mn, fmaxf(cmax[32 + li], cmax[48 + li]));
        if (16 * wid < TK) {
            u32x2 w;
            w[0] = pack_bf2(__builtin_amdgcn_exp2f(sa[0] - mn), __builtin_amdgcn_exp2f(sa[1] - mn));
            w[1] = pack_bf2(__builtin_amdgcn_exp2f(sa[2] - mn), __builtin_amdgcn_exp2f(sa[3] - mn));
            *reinterpret_cast<u32x2*>(Ps + li * PRS + (16 * wid + 4 * g) * 2) = w;
        }
        const float al = __builtin_amdgcn_exp2f(m - mn);          // 0 on the first tile
        m = mn;
        lacc *= al;
#pragma unroll
        for (int d = 0; d < DTW; ++d) oacc[d] *= al;
        __syncthreads();
        bf16x8 pf[TK / 32];
#pragma unroll
        for (int c = 0; c < TK / 32; ++c) {
            const u32x2 lo = *reinterpret_cast<const u32x2*>(Ps + li * PRS + (32 * c + 4 * g) * 2);
            const u32x2 hi = *reinterpret_cast<const u32x2*>(Ps + li * PRS + (32 * c + 16 + 4 * g) * 2);
            pf[c] = __builtin_bit_cast(bf16x8, u32x4{lo[0], lo[1], hi[0], hi[1]});
            lacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[c], lacc, 0, 0, 0);
        }
#pragma unroll
        for (int d = 0; d < DTW; ++d) {
            const int db = wid + 4 * d;
            if (db >= dts) break;
#pragma unroll
            for (int c = 0; c < TK / 32; ++c) {
                const char* va = vrd + 32 * c * RS + 32 * db;
                const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va));
                const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va + 16 * RS));
                const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
                oacc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, u32x4{l2[0], l2[1], h2[0], h2[1]}), pf[c], oacc[d], 0, 0, 0);
            }
        }
    }
    if (h0 + li < p.heads) {
        const long o = slot0 + h0 + li;
#pragma unroll
        for (int d = 0; d < DTW; ++d) {
            const int db = wid + 4 * d;
            if (db < dts) *reinterpret_cast<f32x4*>(p.part_o + o * p.kvp + 16 * db + 4 * g) = oacc[d];
        }
        if (wid == 0 && g == 0) { p.part_ml[o * 2] = m; p.part_ml[o * 2 + 1] = lacc[0]; }
    }
}

// splits of one (sequence, head) -> the head's weighted latent, bf16; 64 latent columns per workgroup
constexpr int MLA_MAX_SPLIT = 128;
__global__ __launch_bounds__(256) void mla_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, int nsplit,
                                                          int heads, int kvp, const float* __restrict__ sink, bf16_t* __restrict__ out) {
    __shared__ float w_sh[MLA_MAX_SPLIT];
    __shared__ float red[4];
    __shared__ float acc_sh[4][64];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int h = blockIdx.x, b = blockIdx.y, d = blockIdx.z * 64 + lane;
    const long base = (long)b * nsplit * heads + h;
    float m = -INFINITY, l = 0.f;
    if (tid < nsplit) { m = part_ml[(base + (long)tid * heads) * 2]; l = part_ml[(base + (long)tid * heads) * 2 + 1]; }
    float M = wave_max(m);
    if (lane == 0) red[wid] = M;
    __syncthreads();
    M = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float sk = sink ? sink[h] : -INFINITY;
    M = fmaxf(M, sk);
    const float w = (m == -INFINITY) ? 0.f : exp2f(m - M);
    if (tid < nsplit) w_sh[tid] = w;
    const float lw = wave_sum(l * w);
    __syncthreads();
    if (lane == 0) red[wid] = lw;
    float a = 0.f;
    for (int s = wid; s < nsplit; s += 4) {
        const float ws = w_sh[s];
        if (ws != 0.f) a = fmaf(part_o[(base + (long)s * heads) * kvp + d], ws, a);     // (an empty split's row is not written)
    }
    acc_sh[wid][lane] = a;
    __syncthreads();
    if (wid == 0) {
        float L = (red[0] + red[1]) + (red[2] + red[3]);
        if (sink) L += exp2f(sk - M);
        out[((long)b * heads + h) * kvp + d] = f2bf(((acc_sh[0][lane] + acc_sh[1][lane]) + (acc_sh[2][lane] + acc_sh[3][lane])) / L);
    }
}

template <int KS, int DT, int NQ>
int launch_prefill(hipStream_t st, const CogsMla& a) {
    static std::atomic<uint64_t> attr_done{0};
    constexpr int lds = 64 * (KS * 64) + 64 * (DT * 32 + 32);
    cogs_ensure_dyn_lds((const void*)mla_prefill_kernel<KS, DT, NQ>, lds, attr_done);
    const int nqt = (a.max_new + 64 * NQ - 1) / (64 * NQ);
    const long grid = (long)nqt * a.heads * a.nseq;
    if (grid > 0x7fffffffL) return COGS_E_INVALID;
    hipLaunchKernelGGL((mla_prefill_kernel<KS, DT, NQ>), dim3((unsigned)grid), dim3(256), lds, st, a, nqt);
    return COGS_LAUNCH_CHECK();
}

template <int TK, int DTW, int PER>
int launch_decode(hipStream_t st, const MlaDecodeArgs& p, int nseq) {
    static std::atomic<uint64_t> attr_done{0};
    const int lds = (TK + 16) * (p.kvw * 2 + 32) + 16 * (TK * 2 + 16) + 64 * 4;
    cogs_ensure_dyn_lds((const void*)mla_decode_kernel<TK, DTW, PER>, 160 * 1024, attr_done);
    hipLaunchKernelGGL((mla_decode_kernel<TK, DTW, PER>), dim3((unsigned)((p.nsplit + 7) / 8 * 8 * p.nht), nseq), dim3(256), lds, st, p);
    return COGS_LAUNCH_CHECK();
}

}  // namespace

int cogs_k_mla_latent(hipStream_t st, int dtype, const CogsMlaLatent& a, int rows) {
    if (rows <= 0) return COGS_OK;
    if (a.qrp % 4 || a.kvp % 4 || a.krc % 2 || a.ldt % 4 || a.dr % 2) return COGS_E_INVALID;
    LatentArgs p;
    p.t = a.t; p.ldt = a.ldt; p.qr = a.qr; p.qrp = a.qrp; p.kvr = a.kvr; p.kvp = a.kvp; p.dr = a.dr; p.krc = a.krc;
    p.own_kv = a.own_kv; p.gate_col = a.gate_col; p.heads = a.heads; p.q_norm = a.q_norm; p.kv_norm = a.kv_norm; p.eps = a.eps;
    p.rope = a.rope; p.rope_pairs = a.rope_pairs; p.rope_first = a.rope_first; p.cq = a.cq; p.gate = a.gate;
    p.seqs = a.seqs; p.rowseq = a.rowseq; p.rowpos = a.rowpos; p.layer_off = a.layer_off;
    if (dtype == COGS_DT_BF16) hipLaunchKernelGGL(mla_latent_kernel<bf16_t>, dim3(rows), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(mla_latent_kernel<float>, dim3(rows), dim3(256), 0, st, p);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_mla_gather(hipStream_t st, int dtype, const CogsSeq* seqs, int nseq, int max_ctx, long layer_off, int kvw, void* out) {
    const int es = dtype == COGS_DT_BF16 ? 2 : 4;
    if (nseq <= 0 || (kvw * es) % 16) return COGS_E_INVALID;
    long g = ((long)max_ctx * (kvw * es / 16) + 1023) / 1024;
    if (g < 1) g = 1;
    if (g > 1024) g = 1024;
    hipLaunchKernelGGL(mla_gather_kernel, dim3((unsigned)g, nseq), dim3(256), 0, st, seqs, layer_off, kvw * es, es, (char*)out);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_head_gemm(hipStream_t st, int dtype, const CogsHeadGemm& a) {
    if (a.B <= 0 || a.heads <= 0 || a.N <= 0 || a.K <= 0) return COGS_E_INVALID;
    HeadGemmArgs p;
    p.X = a.X; p.ldxb = a.ldxb; p.ldxh = a.ldxh; p.W = a.W; p.Y = a.Y; p.ldyb = a.ldyb; p.ldyh = a.ldyh;
    p.B = a.B; p.heads = a.heads; p.N = a.N; p.K = a.K; p.gate = a.gate;
    p.tail = a.tail; p.tail_src = a.tail_src; p.tail_n = a.tail_n;
    if (dtype == COGS_DT_BF16) {
        if (a.N % 16 || a.K % 32 || a.ldxb % 8 || a.ldxh % 8 || a.ldyb % 4 || a.ldyh % 4) return COGS_E_INVALID;
        const int nt = (a.N + a.tail + 15) / 16;
        hipLaunchKernelGGL(head_gemm_bf16_kernel, dim3((nt + 3) / 4, a.heads, (a.B + 15) / 16), dim3(256), 0, st, p);
    } else {
        hipLaunchKernelGGL(head_gemm_f32_kernel, dim3((a.N + a.tail + 3) / 4, a.heads, a.B), dim3(256), 0, st, p);
    }
    return COGS_LAUNCH_CHECK();
}

// attention of every new row over the expanded context (absorbed == 0) or over the cache rows themselves
int cogs_k_mla_attention(hipStream_t st, int dtype, const CogsMla& a) {
    if (a.rows <= 0 || a.nseq <= 0 || a.heads <= 0 || a.dn % 4 || a.dr % 4 || a.dv <= 0) return COGS_E_INVALID;
    const int es = dtype == COGS_DT_BF16 ? 2 : 4;
    if ((a.ldk * es) % 8 || (a.ldkr * es) % 8 || (a.ldv * es) % 8) return COGS_E_INVALID;
    if (dtype == COGS_DT_BF16 && !a.absorbed && a.dn % 8 == 0 && a.dr % 8 == 0 && a.dv % 16 == 0 && a.ldq % 8 == 0 && a.q_head % 8 == 0 &&
        a.q_head >= (a.dn + a.dr + 31) / 32 * 32 && a.ldk % 8 == 0 && a.k_head % 8 == 0 && a.ldkr % 8 == 0 && a.ldv % 8 == 0 &&
        a.v_head % 8 == 0 && a.ldo % 4 == 0 && a.o_head % 4 == 0 && g_cogs_debug.mla_rowwise == 0) {
        const int ks = (a.dn + a.dr + 31) / 32, dt = a.dv / 16;
        if (ks <= 2 && dt <= 4) return launch_prefill<2, 4, 2>(st, a);
        if (ks <= 4 && dt <= 4) return launch_prefill<4, 4, 2>(st, a);
        if (ks <= 4 && dt <= 8) return launch_prefill<4, 8, 2>(st, a);
        if (ks <= 6 && dt <= 8) return launch_prefill<6, 8, 2>(st, a);
        if (ks <= 8 && dt <= 8) return launch_prefill<8, 8, 2>(st, a);
        if (ks <= 8 && dt <= 16) return launch_prefill<8, 16, 1>(st, a);
    }
    if (a.dn + a.dr > RW_DIM || a.dv > 64 * RW_VREG) return COGS_E_UNSUPPORTED;
    if (dtype == COGS_DT_BF16) hipLaunchKernelGGL(mla_rowwise_kernel<bf16_t>, dim3(a.rows, a.heads), dim3(64), 0, st, a);
    else hipLaunchKernelGGL(mla_rowwise_kernel<float>, dim3(a.rows, a.heads), dim3(64), 0, st, a);
    return COGS_LAUNCH_CHECK();
}

bool cogs_k_mla_decode_fits(int kvw, int kvp) {
    return kvw % 32 == 0 && kvp % 16 == 0 && kvp <= 1024 && (32 + 16) * (kvw * 2 + 32) + 16 * (32 * 2 + 16) + 256 <= 160 * 1024 &&
           32 * (kvw / 8) <= 256 * 18;
}

int cogs_k_mla_decode_splits(int nseq, int heads, int max_ctx) {
    const int keys = (int)g_cogs_debug.mla_split_keys;
    int n;
    if (keys > 0) n = (max_ctx + keys - 1) / keys;
    else {
        const int nht = (heads + 15) / 16;
        n = 512 / (nseq * nht);                           // about two workgroups per CU
        const int tiles = (max_ctx + 63) / 64;
        if (n > tiles) n = tiles;
    }
    if (n < 1) n = 1;
    return n > MLA_MAX_SPLIT ? MLA_MAX_SPLIT : n;
}

// one new row per sequence, absorbed queries [seq][heads][kvw]; -> latent sums [seq][heads][kvp]
int cogs_k_mla_decode(hipStream_t st, const CogsMlaDecode& a) {
    if (a.nseq <= 0 || a.nseq > 65535 || a.nsplit < 1 || a.nsplit > MLA_MAX_SPLIT || !cogs_k_mla_decode_fits(a.kvw, a.kvp) || a.kvp % 64 ||
        a.ldq % 8 || a.q_head % 8 || a.heads <= 0) return COGS_E_INVALID;
    MlaDecodeArgs p;
    p.Q = (const bf16_t*)a.Q; p.ldq = a.ldq; p.q_head = a.q_head; p.seqs = a.seqs; p.layer_off = a.layer_off;
    p.kvw = a.kvw; p.kvp = a.kvp; p.heads = a.heads; p.nht = (a.heads + 15) / 16; p.nsplit = a.nsplit;
    p.part_o = a.part; p.part_ml = a.part + (size_t)a.nseq * a.nsplit * a.heads * a.kvp;
    const int dtw = (a.kvp / 16 + 3) / 4, ch64 = 64 * (a.kvw / 8);
    int rc;
    if (dtw <= 2 && ch64 <= 256 * 6) rc = launch_decode<64, 2, 6>(st, p, a.nseq);
    else if (dtw <= 4 && ch64 <= 256 * 10) rc = launch_decode<64, 4, 10>(st, p, a.nseq);
    else if (dtw <= 8 && ch64 <= 256 * 18) rc = launch_decode<64, 8, 18>(st, p, a.nseq);
    else rc = launch_decode<32, 16, 18>(st, p, a.nseq);
    if (rc != COGS_OK) return rc;
    hipLaunchKernelGGL(mla_combine_kernel, dim3(a.heads, a.nseq, a.kvp / 64), dim3(256), 0, st, p.part_o, p.part_ml, a.nsplit, a.heads, a.kvp,
                       a.sink, (bf16_t*)a.out);
    return COGS_LAUNCH_CHECK();
}
