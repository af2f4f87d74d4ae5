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
// The same kernels serve attention whose keys and values are cached per head (cogs_attn_mixer): a cache block per key / value head
// with rows [key | value] takes the place of the latent rows, query heads share a block in groups, there is no shared rotated part,
// and a learned bias per head and distance may be added to the scores. The bias is constant from some distance on, so only the key
// tiles near the diagonal look it up; for the others it is part of the accumulators' start value.
//
// Scores are in log2 units everywhere (the query projection's epilogue multiplies by scale * log2 e before its rounding), so are
// the optional per-head sinks: a sink joins the softmax sum with no key and no value. The optional per-head output gate
// multiplies the finished head row.
//
// Padded sizes (zeros, by the packer): dn = unrotated query/key part, dr = rotated part (multiples of 8), dv = value
// (multiple of 16); a query head is [dn, zeros to a 32-multiple | dr, zeros to a 32-multiple]; a cache row is [c: kvp = 64-multiple | kr:
// 32-multiple] = kvw columns.
#include "common.h"
#include "kernels.h"
#include "debug.h"
#include <type_traits>

namespace {

__device__ __forceinline__ float col_max4(float x) {      // over the lanes {li, li+16, li+32, li+48}, result in all four
    const unsigned xb = __builtin_bit_cast(unsigned, x);
    const auto a = __builtin_amdgcn_permlane16_swap(xb, xb, false, false);
    const float y = fmaxf(__builtin_bit_cast(float, (unsigned)a[0]), __builtin_bit_cast(float, (unsigned)a[1]));
    const unsigned yb = __builtin_bit_cast(unsigned, y);
    const auto b = __builtin_amdgcn_permlane32_swap(yb, yb, false, false);
    return fmaxf(__builtin_bit_cast(float, (unsigned)b[0]), __builtin_bit_cast(float, (unsigned)b[1]));
}

// two softmax weights as MFMA operands: bf16 head and bf16 remainder (together 16 significant bits), packed lower half first
__device__ __forceinline__ void split_weights(float p0, float p1, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf2(p0, p1);
    lo = pack_bf2(p0 - bf_lo(hi), p1 - bf_hi(hi));
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

// y[b][h][n] = sum_k x[b][h][k] W[h][n][k]: up to 16 batch rows are the MFMA columns. A wave owns 16 outputs of one head; KSPLIT:
// a workgroup does, and its waves take every fourth 32-wide step of K (the long K of the value product)
template <bool KSPLIT>
__global__ __launch_bounds__(256) void head_gemm_bf16_kernel(HeadGemmArgs p) {
    __shared__ __attribute__((aligned(16))) f32x4 red[KSPLIT ? 4 : 1][64];
    const int lane = threadIdx.x & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int h = blockIdx.y, b0 = blockIdx.z * 16, b = b0 + li;
    const int n0 = (KSPLIT ? blockIdx.x : blockIdx.x * 4 + wid) * 16;
    const bf16_t* x = reinterpret_cast<const bf16_t*>(p.X) + (long)min(b, p.B - 1) * p.ldxb + h * p.ldxh;
    bf16_t* y = reinterpret_cast<bf16_t*>(p.Y) + (long)min(b, p.B - 1) * p.ldyb + h * p.ldyh;
    if (n0 >= p.N) {
        if (n0 < p.N + p.tail && b < p.B && (!KSPLIT || wid == 0)) {
            const int j0 = n0 - p.N + 4 * g;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (j0 + e < p.tail) y[p.N + j0 + e] = j0 + e < p.tail_n ? x[p.tail_src + j0 + e] : (bf16_t)0;
        }
        return;
    }
    const bf16_t* w = reinterpret_cast<const bf16_t*>(p.W) + ((long)h * p.N + n0 + li) * p.K + 8 * g;
    x += 8 * g;
    constexpr int STEP = KSPLIT ? 4 : 1;
    const int nk = p.K >> 5;
    f32x4 a0 = {0.f, 0.f, 0.f, 0.f}, a1 = a0;
    for (int k = KSPLIT ? wid : 0; k < nk; k += 4 * STEP) {          // four 32-wide steps in flight; steps past the end are not multiplied
        u32x4 wf[4], xf[4];
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            const int o = 32 * min(k + STEP * s, nk - 1);
            wf[s] = *reinterpret_cast<const u32x4*>(w + o);
            xf[s] = *reinterpret_cast<const u32x4*>(x + o);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            if (k + STEP * s >= nk) break;
            f32x4& a = (s & 1) ? a1 : a0;
            a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf[s]), __builtin_bit_cast(bf16x8, xf[s]), a, 0, 0, 0);
        }
    }
    a0 += a1;
    if constexpr (KSPLIT) {
        red[wid][lane] = a0;
        __syncthreads();
        if (wid) return;
        a0 = (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]);
    }
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
    for (int d = lane; d < p.dn + p.dr; d += 64) qs[d] = ld_f<T>(q + (d < p.dn ? d : p.q_rot + d - p.dn));
    __syncthreads();
    const T *K, *KR, *V;
    if (p.kvw) {
        K = reinterpret_cast<const T*>(s.cache) + (p.layer_off + (long)(h / p.rep) * p.kvw) * s.max_len;
        V = K + p.v_col;
        KR = K;
    } else if (p.absorbed) {
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
        const float sc = (a[0] + a[1]) + (a[2] + a[3]);
        return p.bias ? sc + p.bias[(long)h * p.nb + min(nkeys - 1 - j, p.nb - 1)] : sc;
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
// 4 waves x 32 query rows of one (sequence, head) against 64-key tiles. Staging as in attn.hip's prompt kernel: a tile's pieces
// (1 KiB = 64 lanes x 16 bytes) go global -> LDS by LDS-DMA into a double buffer, one tile ahead, one barrier per tile. Keys come
// from two places -- the head's expanded part and the rotated part all heads share -- so a K tile is two LDS regions of KN and KR
// 32-dimension steps. LDS-DMA writes lane-linear images: the bank swizzles live on the source address.
//   scores transposed, S^T = K.Q^T, key rows permuted so that a lane's registers of blocks 2u, 2u+1 are the B operand of the
//   u-th 32-key step of O^T = V^T.P^T; the accumulator starts at minus the running reference, so P = exp2(acc); the reference
//   moves only when a score passes it by 2^THR (the sums stay far inside fp32);
//   a weight enters the products as two bf16 terms, head and remainder, so that it is not rounded to 16 bits on its way to V;
//   the softmax sum is one more MFMA per step with an all-ones A operand, i.e. the sum of exactly the weights that multiply V.
// Columns past dn / dr / dv hold copies of real data: the query's are zero, and value tiles past dv are not stored.
// KR = 0: keys and values per head from the cache (rows [key | value] of block h / rep), with the optional distance bias. Distances a
// tile spans are a window of 191 entries, staged in LDS one tile ahead; a tile whose distances are all past the table's end takes
// the last entry with the accumulators' start value.
constexpr float MLA_THR = 6.f;
constexpr int MLA_WIN = 192;             // floats of a bias window

// 16-byte-chunk XOR of row `row` for rows of `chunks` chunks: 16 rows {8 a + b (+ 4 c)} of a fragment read land in different banks
template <int CHUNKS> __device__ __forceinline__ int mla_kswz(int row) {
    if constexpr (CHUNKS % 16 == 0) return (row & 3) | (((row >> 3) & 3) << 2);
    else if constexpr (CHUNKS % 8 == 0) return ((row >> 1) & 1) | (((row >> 3) & 3) << 1);
    else return (row >> 3) & 3;
}
// 32-byte-unit XOR of a V row of DT units: the (row & 3, row bit 3) classes of a transposing read land in different banks
template <int DT> __device__ __forceinline__ int mla_vswz(int row) {
    const int b3 = (row >> 3) & 1;
    if constexpr (DT % 8 == 0) return (row & 3) | (b3 << 2);
    else if constexpr (DT % 4 == 0) return ((row >> 1) & 1) | (b3 << 1);
    else return b3;
}

template <int KN, int KR, int DT, int WGS>
__global__ __launch_bounds__(256, WGS) void mla_prefill_kernel(CogsMla p, int nqt, int group) {
    constexpr int NQ = 2, KS = KN + KR;
    constexpr bool HEADS = KR == 0;
    constexpr int N_LDS = 64 * KN * 64, R_LDS = 64 * KR * 64, V_LDS = 64 * DT * 32, BUF = N_LDS + R_LDS + V_LDS;
    constexpr int PV = DT / 2;                    // V pieces per wave (K: KN and KR)
    static_assert(DT % 2 == 0, "whole pieces per wave");
    extern __shared__ __attribute__((aligned(16))) char smem[];

    const int tid = threadIdx.x, lane = tid & 63;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, g = lane >> 4;
    // launch order -> (sequence, head) and query tile. An XCD gets a contiguous run, `group` (sequence, head) pairs at a time (their
    // K / V meet in its L2), long query tiles first; where a group is two waves of one workgroup per CU (<= 64), the second
    // wave runs short to long, so that the two workgroups of a CU add up to the same length everywhere
    int qt, pair;
    {
        const int total = gridDim.x, xcd = blockIdx.x & 7, q = total >> 3, r = total & 7;
        const int bid = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (blockIdx.x >> 3);
        const int per = group * nqt, grp = bid / per, np = total / nqt;
        int i = bid - grp * per;
        const int gsz = min(group, np - grp * group), n = gsz * nqt;
        if (n <= 64 && i >= 32) i = n - 1 - (i - 32);
        qt = nqt - 1 - i / gsz;
        pair = grp * group + i % gsz;
    }
    const int h = pair % p.heads;
    const CogsSeq s = p.seqs[pair / p.heads];
    const int q0 = qt * 128;
    if (q0 >= s.len) return;

    const bf16_t* Q = reinterpret_cast<const bf16_t*>(p.Q) + (long)s.row0 * p.ldq + (long)h * p.q_head;
    const bf16_t *K, *KRp = nullptr, *V;
    if constexpr (HEADS) {
        K = reinterpret_cast<const bf16_t*>(s.cache) + (p.layer_off + (long)(h / p.rep) * p.kvw) * s.max_len;
        V = K + p.v_col;
    } else {
        K = reinterpret_cast<const bf16_t*>(p.K) + (long)s.ctx0 * p.ldk + (long)h * p.k_head;
        KRp = reinterpret_cast<const bf16_t*>(p.KR) + (long)s.ctx0 * p.ldkr;
        V = reinterpret_cast<const bf16_t*>(p.V) + (long)s.ctx0 * p.ldv + (long)h * p.v_head;
    }

    bf16x8 qf[NQ][KS];
    int qpos[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        const int rc = min(q0 + wid * 32 + 16 * i + li, s.len - 1);
        qpos[i] = s.pos0 + rc;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int kk = k < KN ? 32 * k : p.q_rot + 32 * (k - KN);
            u32x4 v = {0, 0, 0, 0};
            if (k < KN ? 32 * k < p.q_rot : kk < p.q_head) v = *reinterpret_cast<const u32x4*>(Q + (long)rc * p.ldq + kk + 8 * g);
            qf[i][k] = __builtin_bit_cast(bf16x8, v);
        }
    }
    const bool wave_active = q0 + wid * 32 < s.len;
    const int wave_hi = s.pos0 + min(q0 + wid * 32 + 31, s.len - 1);               // last position of the wave's rows
    const int kend = s.pos0 + min(q0 + 128, s.len);                                 // keys the workgroup needs
    const int nt = (kend + 63) >> 6;
    const int p0 = s.pos0 + q0;                                                     // position of the workgroup's first row
    float b_far = 0.f;
    int t_far = 0;                                                                  // tiles [0, t_far) lie past the bias table's end
    float* const win = reinterpret_cast<float*>(smem + 2 * BUF);
    if constexpr (HEADS) {
        if (p.bias) {
            b_far = p.bias[(long)h * p.nb + p.nb - 1];
            const int d = p0 - 62 - p.nb;                                           // kb <= p0 - 63 - (nb - 1)
            t_far = d >= 0 ? (d >> 6) + 1 : 0;
        } else t_far = nt;
    }

    f32x4 oacc[DT][NQ], lacc[NQ];
    float m_ref[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        m_ref[i] = 0.f;
        lacc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < DT; ++d) oacc[d][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const bf16x8 ones = __builtin_bit_cast(bf16x8, u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u});

    // staging: wave w issues pieces w, w + 4, ... of each region; byte offsets from the tile's first row
    const unsigned smem_lds = (unsigned)(size_t)(__attribute__((address_space(3))) char*)smem;
    const int nkc = p.dn >> 3, nrc = p.dr >> 3, nvc = p.dv >> 3;
    auto k_slot = [&](int i, int& row, int& chunk) {
        constexpr int CH = KN * 4;
        const int id = 64 * (wid + 4 * i) + lane;
        row = id / CH;
        chunk = min((id % CH) ^ mla_kswz<CH>(row), nkc - 1);
    };
    auto r_slot = [&](int i, int& row, int& chunk) {
        constexpr int CH = KR > 0 ? KR * 4 : 4;
        const int id = 64 * (wid + 4 * i) + lane;
        row = id / CH;
        chunk = min((id % CH) ^ mla_kswz<CH>(row), nrc - 1);
    };
    auto v_slot = [&](int i, int& row, int& chunk) {
        constexpr int CH = DT * 2;
        const int id = 64 * (wid + 4 * i) + lane, sl = id % CH;
        row = id / CH;
        chunk = min((((sl >> 1) ^ mla_vswz<DT>(row)) << 1) | (sl & 1), nvc - 1);
    };
    int k_off[KN], r_off[KR + 1], v_off[PV];
#pragma unroll
    for (int i = 0; i < KN; ++i) { int row, c; k_slot(i, row, c); k_off[i] = (row * (int)p.ldk + c * 8) * 2; }
    if constexpr (!HEADS) {
#pragma unroll
        for (int i = 0; i < KR; ++i) { int row, c; r_slot(i, row, c); r_off[i] = (row * (int)p.ldkr + c * 8) * 2; }
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) { int row, c; v_slot(i, row, c); v_off[i] = (row * (int)p.ldv + c * 8) * 2; }
    auto uniform_ptr = [](const bf16_t* q) -> const bf16_t* {
        const unsigned long long v = (unsigned long long)q;
        const unsigned lo = __builtin_amdgcn_readfirstlane((unsigned)v), hi = __builtin_amdgcn_readfirstlane((unsigned)(v >> 32));
        return (const bf16_t*)(((unsigned long long)hi << 32) | lo);
    };
    // (inline assembly for the reason attn_vit.hip gives; the build checks that nothing else in this kernel touches M0)
    auto dma16 = [&](const bf16_t* base, int off_bytes, unsigned lds) {
        asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2" :: "s"(lds), "v"(off_bytes), "s"(base) : "memory");
    };
    auto issue_tile = [&](int t) {
        const int kb = t * 64, valid = kend - kb;                      // >= 1; rows past the end repeat the last one (masked)
        const bf16_t* kp = uniform_ptr(K + (long)kb * p.ldk);
        const bf16_t* rp = HEADS ? nullptr : uniform_ptr(KRp + (long)kb * p.ldkr);
        const bf16_t* vp = uniform_ptr(V + (long)kb * p.ldv);
        const unsigned st = __builtin_amdgcn_readfirstlane(smem_lds + (t & 1) * BUF);
        const bool ragged = valid < 64;
#pragma unroll
        for (int i = 0; i < KN; ++i) {
            int o = k_off[i];
            if (ragged) { int row, c; k_slot(i, row, c); o -= max(row - (valid - 1), 0) * (int)p.ldk * 2; }
            dma16(kp, o, st + (wid + 4 * i) * 1024);
        }
        if constexpr (!HEADS) {
#pragma unroll
            for (int i = 0; i < KR; ++i) {
                int o = r_off[i];
                if (ragged) { int row, c; r_slot(i, row, c); o -= max(row - (valid - 1), 0) * (int)p.ldkr * 2; }
                dma16(rp, o, st + N_LDS + (wid + 4 * i) * 1024);
            }
        }
#pragma unroll
        for (int i = 0; i < PV; ++i) {
            int o = v_off[i];
            if (ragged) { int row, c; v_slot(i, row, c); o -= max(row - (valid - 1), 0) * (int)p.ldv * 2; }
            dma16(vp, o, st + N_LDS + R_LDS + (wid + 4 * i) * 1024);
        }
    };

    // bias window of tile t: entry i is distance p0 - 63 - 64 t + i (queries below p0 + 128, keys 64 t .. 64 t + 63)
    auto stage_window = [&](int t) {
        if constexpr (HEADS)
            if (t >= t_far && tid < MLA_WIN)
                win[(t & 1) * MLA_WIN + tid] = p.bias[(long)h * p.nb + min(max(p0 - 63 - 64 * t + tid, 0), p.nb - 1)];
    };

    const int krow0 = 8 * (li >> 2) + (li & 3);
    const int vr = 8 * g + (li >> 2);                  // + 32 u (+ 4): mla_vswz is the same for all of them
    const int v_sw = mla_vswz<DT>(vr);
    const int v_base = vr * (DT * 32) + (li & 3) * 8;

    auto process_tile = [&](const int t, auto masked_tag, auto first_tag, auto near_tag) {
        constexpr bool MASKED = decltype(masked_tag)::value, FIRST = decltype(first_tag)::value;
        constexpr bool NEAR = HEADS && decltype(near_tag)::value;
        const int kb = t * 64;
        if (!wave_active || (MASKED && kb > wave_hi)) return;
        const char* Ns = smem + (t & 1) * BUF;
        const char* Rs = Ns + N_LDS;
        const char* Vs = Rs + R_LDS;
        f32x4 sacc[4][NQ];
        __builtin_amdgcn_s_setprio(0);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int krow = 32 * (u >> 1) + 4 * (u & 1) + krow0;
            const int nsw = mla_kswz<KN * 4>(krow), rsw = HEADS ? 0 : mla_kswz<KR * 4>(krow);
            f32x4 start[NQ];
#pragma unroll
            for (int i = 0; i < NQ; ++i) {
                const float nm = HEADS && !NEAR ? b_far - m_ref[i] : -m_ref[i];
                start[i] = f32x4{nm, nm, nm, nm};
                if constexpr (NEAR) {
                    const float* b = win + (t & 1) * MLA_WIN + (qpos[i] - p0 + 63 - (32 * (u >> 1) + 8 * g + 4 * (u & 1)));
#pragma unroll
                    for (int r = 0; r < 4; ++r) start[i][r] += b[-r];
                }
            }
#pragma unroll
            for (int k = 0; k < KS; ++k) {
                const char* a = k < KN ? Ns + krow * (KN * 64) + (((4 * k + g) ^ nsw) << 4)
                                       : Rs + krow * (KR * 64) + (((4 * (k - KN) + g) ^ rsw) << 4);
                const bf16x8 kf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(a));
#pragma unroll
                for (int i = 0; i < NQ; ++i)
                    sacc[u][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i][k], k == 0 ? start[i] : sacc[u][i], 0, 0, 0);
            }
        }
        if constexpr (!MASKED && !NEAR && KS >= 2) {   // 4 KS reads, 8 KS MFMAs: six reads lead, then a read per pair of MFMAs
            __builtin_amdgcn_sched_group_barrier(0x100, 6, 0);
#pragma unroll
            for (int i = 0; i < 4 * KS - 6; ++i) {
                __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
                __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
            }
            __builtin_amdgcn_sched_group_barrier(0x008, 12, 0);
        }
        __builtin_amdgcn_s_setprio(1);
        bf16x8 pf[2][NQ][2];                           // [32-key step][row group][head, remainder]
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            float d = -INFINITY;
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if constexpr (MASKED)
                        if (kb + 32 * (u >> 1) + 8 * g + 4 * (u & 1) + r > qpos[i]) sacc[u][i][r] = -INFINITY;
                    d = fmaxf(d, sacc[u][i][r]);
                }
            if constexpr (FIRST) {                     // key 0 is visible to every row: finite
                d = col_max4(d);
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sacc[u][i][r] -= d;
                m_ref[i] = d;
            } else if (__any(d > MLA_THR)) {
                const float dr = col_max4(d), dd = dr > MLA_THR ? dr : 0.f;
                const float al = __builtin_amdgcn_exp2f(-dd);
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int r = 0; r < 4; ++r) sacc[u][i][r] -= dd;
                lacc[i] *= al;
#pragma unroll
                for (int e = 0; e < DT; ++e) oacc[e][i] *= al;
                m_ref[i] += dd;
            }
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                u32x4 w, x;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    uint32_t hi, lo;
                    split_weights(__builtin_amdgcn_exp2f(sacc[2 * u + (e >> 1)][i][2 * (e & 1)]),
                                  __builtin_amdgcn_exp2f(sacc[2 * u + (e >> 1)][i][2 * (e & 1) + 1]), hi, lo);
                    w[e] = hi; x[e] = lo;
                }
                pf[u][i][0] = __builtin_bit_cast(bf16x8, w);
                pf[u][i][1] = __builtin_bit_cast(bf16x8, x);
            }
        }
        __builtin_amdgcn_s_setprio(0);
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < NQ; ++i)
#pragma unroll
                for (int x = 0; x < 2; ++x) lacc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[u][i][x], lacc[i], 0, 0, 0);
#pragma unroll
        for (int d = 0; d < DT; ++d)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const char* va = Vs + u * 32 * (DT * 32) + v_base + ((d ^ v_sw) << 5);
                const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va));
                const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va + 4 * (DT * 32)));
                const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
                const bf16x8 vf = __builtin_bit_cast(bf16x8, u32x4{l2[0], l2[1], h2[0], h2[1]});
#pragma unroll
                for (int x = 0; x < 2; ++x)
#pragma unroll
                    for (int i = 0; i < NQ; ++i) oacc[d][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[u][i][x], oacc[d][i], 0, 0, 0);
            }
        if constexpr (!MASKED && DT >= 4) {            // 4 DT transposing reads, 8 + 8 DT MFMAs: eight reads lead
            __builtin_amdgcn_sched_group_barrier(0x100, 8, 0);
            __builtin_amdgcn_sched_group_barrier(0x008, 8, 0);
#pragma unroll
            for (int i = 0; i < DT - 2; ++i) {
                __builtin_amdgcn_sched_group_barrier(0x008, 8, 0);
                __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
            }
            __builtin_amdgcn_sched_group_barrier(0x008, 16, 0);
        }
    };

    // tiles [0, t_mid) lie left of the diagonal of every row
    const int t_mid = min((s.pos0 + q0 + 1) >> 6, nt);
    issue_tile(0);
    stage_window(0);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
#pragma unroll
    for (int i = 0; i < NQ; ++i)
#pragma unroll
        for (int k = 0; k < KS; ++k) asm volatile("" : "+v"(qf[i][k]));          // Q loads complete before the loop
    if constexpr (HEADS) asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    auto tile_tail = [&] {
        // the next tile has landed for this wave, behind the barrier for every wave, and nobody reads this one any more
        if constexpr (HEADS) asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
    };
    auto next_tile = [&](int t) {
        if (t >= nt) return;
        issue_tile(t);
        stage_window(t);
    };
    typedef std::true_type yes;
    typedef std::false_type no;
    next_tile(1);
    // masked tiles look the bias up, unless there is none
    const bool no_bias = HEADS && t_far >= nt;
    if (t_mid <= 0) {
        if (no_bias) process_tile(0, yes{}, yes{}, no{});
        else process_tile(0, yes{}, yes{}, yes{});
    } else if (!HEADS || 0 < t_far) process_tile(0, no{}, yes{}, no{});
    else process_tile(0, no{}, yes{}, yes{});
    tile_tail();
    int t = 1;
    const int t_plain = HEADS ? min(t_mid, t_far) : t_mid;
    for (; t < t_plain; ++t) {
        next_tile(t + 1);
        process_tile(t, no{}, no{}, no{});
        tile_tail();
    }
    if constexpr (HEADS) {
        for (; t < t_mid; ++t) {
            next_tile(t + 1);
            process_tile(t, no{}, no{}, yes{});
            tile_tail();
        }
    }
    for (; t < nt; ++t) {
        next_tile(t + 1);
        if (no_bias) process_tile(t, yes{}, no{}, no{});
        else process_tile(t, yes{}, no{}, yes{});
        tile_tail();
    }

    const int dt = p.dv >> 4;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        const int qrow = q0 + wid * 32 + 16 * i + li;
        if (qrow >= s.len) continue;
        float f = 1.f / (lacc[i][0] + (p.sink ? exp2f(p.sink[h] - m_ref[i]) : 0.f));
        const long row = s.row0 + qrow;
        if (p.gate) f *= p.gate[row * p.heads + h];
        bf16_t* O = reinterpret_cast<bf16_t*>(p.O) + row * p.ldo + (long)h * p.o_head + 4 * g;
#pragma unroll
        for (int d = 0; d < DT; ++d)
            if (d < dt) st4_f<bf16_t>(O + 16 * d, oacc[d][i] * f);
    }
}

// ------------------------------------------------------------------------------------------------ decode attention (bf16)
// One new row per sequence. Workgroup = (split of the keys, 16 heads, sequence). A tile of 32 cache rows is one contiguous run in
// memory; it goes through registers into LDS (the next tile's loads are in flight meanwhile) and is read twice there: as K rows
// (A operand of S^T = C.Q^T; waves share the product as 2 key blocks x 2 halves of the row) and transposed as V (A operand of
// O^T = C^T.P^T; wave w owns the latent columns 16 (w + 4 i)). The four partial score tiles meet in LDS in the accumulators' own
// lane layout: every wave adds the halves of both blocks and has all 32 weights of its 16 query columns as the B operand.
struct MlaDecodeArgs {
    const bf16_t* Q; long ldq; int q_head;
    const CogsSeq* seqs; long layer_off;
    int kvw, kcols, vcol, kvp;              // cache row: columns [0, kcols) meet the query, [vcol, vcol + kvp) are summed
    int heads, rep, groups, nht, nsplit;    // rep query heads read one cache block, `groups` blocks per sequence
    const float* bias; int nb;              // [heads][nb] added at distance min(n, nb - 1), or null
    float* part_o; float* part_ml;          // [seq][split][head][kvp] relative to part_ml[..][0]; [..][2] = (max, sum)
};

template <int DTW, int PER, int WGS>
__global__ __launch_bounds__(256, WGS) void mla_decode_kernel(MlaDecodeArgs p) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    constexpr int TK = 32;
    const int RS = p.kvw * 2 + 32;                               // an odd multiple of 32 bytes (kvw % 32 == 0)
    f32x4* const Sx = reinterpret_cast<f32x4*>(smem);            // [key block][row half][lane]
    char* const Ks = smem + 4 * 64 * 16;
    char* const Qs = Ks + TK * RS;

    const int tid = threadIdx.x, lane = tid & 63;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, g = lane >> 4;
    // the head tiles of a split sit 8 apart in the launch order = on one XCD: its L2 serves the second and later readers
    const int bid = blockIdx.x, slot = bid & 7, rest = bid >> 3;
    const int ht = rest % p.nht, split = (rest / p.nht) * 8 + slot;
    if (split >= p.nsplit) return;
    const int b = blockIdx.y / p.groups, grp = blockIdx.y - b * p.groups, h0 = grp * p.rep + ht * 16, h1 = (grp + 1) * p.rep;
    const CogsSeq s = p.seqs[b];
    const int kend = s.pos0 + 1;
    const unsigned nt_all = (unsigned)(kend + TK - 1) / TK;
    const int t_begin = (int)(nt_all * (unsigned)split / (unsigned)p.nsplit);
    const int t_end = (int)(nt_all * (unsigned)(split + 1) / (unsigned)p.nsplit);
    const long slot0 = ((long)b * p.nsplit + split) * p.heads;
    if (t_begin >= t_end) {                                        // nothing to do: an empty partial
        if (tid < 16 && h0 + tid < h1) { p.part_ml[(slot0 + h0 + tid) * 2] = -INFINITY; p.part_ml[(slot0 + h0 + tid) * 2 + 1] = 0.f; }
        return;
    }
    const char* cache = s.cache + (p.layer_off + (long)grp * p.kvw) * s.max_len * 2;
    const int row_bytes = p.kvw * 2, nch = p.kvw >> 3, nqc = p.kcols >> 3;      // 16-byte chunks of a row
    const int tile_chunks = TK * nch;
    const int dr_row = 256 / nch, dr_c = 256 % nch;

    u32x4 reg[PER];
    auto load_tile = [&](int t) {
        const char* base = cache + (long)t * TK * row_bytes;
        const int lim = min(TK, kend - t * TK) * nch - 1;           // chunks past the end repeat the last one (masked)
#pragma unroll
        for (int i = 0; i < PER; ++i)
            reg[i] = *reinterpret_cast<const u32x4*>(base + min(tid + 256 * i, lim) * 16);
    };
    load_tile(t_begin);
    const int row_t = tid / nch, c_t = tid - row_t * nch;
    {
        int r = row_t, c = c_t;
#pragma unroll 1
        while (r < 16) {
            u32x4 v = {0, 0, 0, 0};
            if (h0 + r < h1 && c < nqc) v = *reinterpret_cast<const u32x4*>(p.Q + (long)b * p.ldq + (long)(h0 + r) * p.q_head + c * 8);
            *reinterpret_cast<u32x4*>(Qs + r * RS + c * 16) = v;
            r += dr_row; c += dr_c;
            if (c >= nch) { c -= nch; ++r; }
        }
    }
    const int ks = p.kcols >> 5, dts = p.kvp >> 4, kh = (ks + 1) >> 1;
    const int k_lo = (wid >> 1) ? kh : 0, k_hi = (wid >> 1) ? ks : kh;
    f32x4 oacc[DTW], lacc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int d = 0; d < DTW; ++d) oacc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY;
    const bf16x8 ones = __builtin_bit_cast(bf16x8, u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u});
    const char* const qrd = Qs + li * RS + 16 * g;
    const char* const krd = Ks + (16 * (wid & 1) + li) * RS + 16 * g;
    const char* const vrd = Ks + (4 * g + (li >> 2)) * RS + (li & 3) * 8 + 32 * wid + p.vcol * 2;
    const float* const bias = p.bias ? p.bias + (long)min(h0 + li, h1 - 1) * p.nb : nullptr;
    const float b_far = bias ? bias[p.nb - 1] : 0.f;

    for (int t = t_begin; t < t_end; ++t) {
        __syncthreads();                                          // the previous tile's transposed reads are done
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
        f32x4 bias0 = {b_far, b_far, b_far, b_far}, bias1 = bias0;
        if (bias && s.pos0 - t * TK - (TK - 1) < p.nb - 1) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = s.pos0 - t * TK - 4 * g - r;
                bias0[r] = bias[min(max(d, 0), p.nb - 1)];
                bias1[r] = bias[min(max(d - 16, 0), p.nb - 1)];
            }
        }
        {
            f32x4 acc[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[e] = f32x4{0.f, 0.f, 0.f, 0.f};
            int k = k_lo;
#pragma unroll 1
            for (; k + 3 < k_hi; k += 4) {
                u32x4 kf[4], qv[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    kf[e] = *reinterpret_cast<const u32x4*>(krd + 64 * (k + e));
                    qv[e] = *reinterpret_cast<const u32x4*>(qrd + 64 * (k + e));
                }
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    acc[e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kf[e]), __builtin_bit_cast(bf16x8, qv[e]), acc[e], 0, 0, 0);
            }
#pragma unroll 1
            for (; k < k_hi; ++k)
                acc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(krd + 64 * k)),
                                                                 __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(qrd + 64 * k)), acc[0], 0, 0, 0);
            Sx[((wid & 1) * 2 + (wid >> 1)) * 64 + lane] = (acc[0] + acc[1]) + (acc[2] + acc[3]);
        }
        __syncthreads();
        f32x4 s0 = Sx[lane] + Sx[64 + lane] + bias0, s1 = Sx[128 + lane] + Sx[192 + lane] + bias1;
        float tm = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if (4 * g + r >= nvalid) s0[r] = -INFINITY;
            if (16 + 4 * g + r >= nvalid) s1[r] = -INFINITY;
            tm = fmaxf(tm, fmaxf(s0[r], s1[r]));
        }
        const float mn = fmaxf(m, col_max4(tm));                  // finite: the tile's first key exists
        const float al = __builtin_amdgcn_exp2f(m - mn);          // 0 on the first tile
        lacc *= al;
#pragma unroll
        for (int d = 0; d < DTW; ++d) oacc[d] *= al;
        m = mn;
        uint32_t w[4], x[4];                                      // head and remainder of the weights (see the prompt kernel)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            split_weights(__builtin_amdgcn_exp2f(s0[2 * e] - mn), __builtin_amdgcn_exp2f(s0[2 * e + 1] - mn), w[e], x[e]);
            split_weights(__builtin_amdgcn_exp2f(s1[2 * e] - mn), __builtin_amdgcn_exp2f(s1[2 * e + 1] - mn), w[2 + e], x[2 + e]);
        }
        const bf16x8 ph = __builtin_bit_cast(bf16x8, u32x4{w[0], w[1], w[2], w[3]}), pl = __builtin_bit_cast(bf16x8, u32x4{x[0], x[1], x[2], x[3]});
        lacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, ph, lacc, 0, 0, 0);
        lacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pl, lacc, 0, 0, 0);
        // (no branch for columns past kvp: such a read stays inside Ks + Qs, and its accumulator is not stored)
#pragma unroll
        for (int d = 0; d < DTW; ++d) {
            const char* va = vrd + 128 * d;
            const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va));
            const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) i16x4*)(va + 16 * RS));
            const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
            const bf16x8 vf = __builtin_bit_cast(bf16x8, u32x4{l2[0], l2[1], h2[0], h2[1]});
            oacc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, oacc[d], 0, 0, 0);
            oacc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, oacc[d], 0, 0, 0);
        }
    }
    if (h0 + li < h1) {
        const long o = slot0 + h0 + li;
#pragma unroll
        for (int d = 0; d < DTW; ++d) {
            const int db = wid + 4 * d;
            if (db < dts) *reinterpret_cast<f32x4*>(p.part_o + o * p.kvp + 16 * db + 4 * g) = oacc[d];
        }
        if (wid == 0 && g == 0) { p.part_ml[o * 2] = m; p.part_ml[o * 2 + 1] = lacc[0]; }
    }
}

// splits of one (sequence, head) -> the head's weighted latent, bf16; 64 latent columns per workgroup, wave w sums every fourth split
constexpr int MLA_MAX_SPLIT = 256;
__global__ __launch_bounds__(256) void mla_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, int nsplit,
                                                          int heads, int kvp, const float* __restrict__ sink, bf16_t* __restrict__ out,
                                                          long ldo, int o_head) {
    __shared__ float w_sh[MLA_MAX_SPLIT];
    __shared__ float red[4];
    __shared__ float acc_sh[4][64];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int h = blockIdx.x, b = blockIdx.y, d = blockIdx.z * 64 + lane;
    const long base = (long)b * nsplit * heads + h;
    // the first 16 partial rows of this wave are requested before the weights are known (an empty split's row holds anything: its
    // weight is tested, not multiplied)
    const float* po = part_o + base * kvp + min(d, kvp - 1);
    const long stride = (long)heads * kvp;
    float v[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) v[i] = po[(long)min(wid + 4 * i, nsplit - 1) * stride];
    float m = -INFINITY, l = 0.f;
    if (tid < nsplit) { m = part_ml[(base + (long)tid * heads) * 2]; l = part_ml[(base + (long)tid * heads) * 2 + 1]; }
    float M = wave_max(m);
    if (lane == 0) red[wid] = M;
    __syncthreads();
    M = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float sk = sink ? sink[h] : -INFINITY;
    M = fmaxf(M, sk);
    const float w = (m == -INFINITY) ? 0.f : exp2f(m - M);
    w_sh[tid] = w;
    const float lw = wave_sum(l * w);
    __syncthreads();
    if (lane == 0) red[wid] = lw;
    float a = 0.f;
    for (int s0 = 0; s0 < nsplit; s0 += 64) {
        if (s0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) v[i] = po[(long)min(s0 + wid + 4 * i, nsplit - 1) * stride];
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int sp = s0 + wid + 4 * i;
            const float ws = sp < nsplit ? w_sh[sp] : 0.f;
            a += ws != 0.f ? v[i] * ws : 0.f;
        }
    }
    acc_sh[wid][lane] = a;
    __syncthreads();
    if (wid == 0 && d < kvp) {
        float L = (red[0] + red[1]) + (red[2] + red[3]);
        if (sink) L += exp2f(sk - M);
        out[b * ldo + (long)h * o_head + d] = f2bf(((acc_sh[0][lane] + acc_sh[1][lane]) + (acc_sh[2][lane] + acc_sh[3][lane])) / L);
    }
}

template <int KN, int KR, int DT, int WGS>
int launch_prefill(hipStream_t st, const CogsMla& a) {
    static std::atomic<uint64_t> attr_done{0};
    constexpr int lds = 2 * (64 * KN * 64 + 64 * KR * 64 + 64 * DT * 32) + (KR == 0 ? 2 * MLA_WIN * 4 : 0);
    cogs_ensure_dyn_lds((const void*)mla_prefill_kernel<KN, KR, DT, WGS>, lds, attr_done);
    const int nqt = (a.max_new + 127) / 128;
    const long grid = (long)nqt * a.heads * a.nseq;
    if (grid > 0x7fffffffL) return COGS_E_INVALID;
    const int group = nqt >= 64 ? 1 : 64 / nqt;
    hipLaunchKernelGGL((mla_prefill_kernel<KN, KR, DT, WGS>), dim3((unsigned)grid), dim3(256), lds, st, a, nqt, group);
    return COGS_LAUNCH_CHECK();
}

template <int DTW, int PER, int WGS>
int launch_decode(hipStream_t st, const MlaDecodeArgs& p, int nblk) {
    static std::atomic<uint64_t> attr_done{0};
    const int lds = 48 * (p.kvw * 2 + 32) + 4 * 64 * 16;
    cogs_ensure_dyn_lds((const void*)mla_decode_kernel<DTW, PER, WGS>, 160 * 1024, attr_done);
    hipLaunchKernelGGL((mla_decode_kernel<DTW, PER, WGS>), dim3((unsigned)((p.nsplit + 7) / 8 * 8 * p.nht), nblk), dim3(256), lds, st, p);
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
        if (a.K >= 256) hipLaunchKernelGGL(head_gemm_bf16_kernel<true>, dim3(nt, a.heads, (a.B + 15) / 16), dim3(256), 0, st, p);
        else hipLaunchKernelGGL(head_gemm_bf16_kernel<false>, dim3((nt + 3) / 4, a.heads, (a.B + 15) / 16), dim3(256), 0, st, p);
    } else {
        hipLaunchKernelGGL(head_gemm_f32_kernel, dim3((a.N + a.tail + 3) / 4, a.heads, a.B), dim3(256), 0, st, p);
    }
    return COGS_LAUNCH_CHECK();
}

// attention of every new row over the expanded context (absorbed == 0) or over the cache rows themselves
int cogs_k_mla_attention(hipStream_t st, int dtype, const CogsMla& a) {
    if (a.rows <= 0 || a.nseq <= 0 || a.heads <= 0 || a.dn % 4 || a.dr % 4 || a.dv <= 0) return COGS_E_INVALID;
    const int es = dtype == COGS_DT_BF16 ? 2 : 4;
    if (a.kvw) {
        if (a.rep <= 0 || a.heads % a.rep || a.dr || a.ldk != a.kvw || a.ldv != a.kvw || (a.bias && a.nb <= 0)) return COGS_E_INVALID;
    } else if (a.bias) return COGS_E_INVALID;
    if ((a.ldk * es) % 8 || (a.ldkr * es) % 8 || (a.ldv * es) % 8) return COGS_E_INVALID;
    if (dtype == COGS_DT_BF16 && a.kvw && a.dn % 32 == 0 && a.dv % 16 == 0 && a.v_col % 8 == 0 && a.kvw % 8 == 0 && a.ldq % 8 == 0 &&
        a.q_head % 32 == 0 && a.q_head >= a.dn && a.q_rot == a.q_head && a.ldo % 4 == 0 && a.o_head % 4 == 0 && g_cogs_debug.mla_rowwise == 0 &&
        a.kvw < (1 << 23)) {
        const int kn = a.dn / 32, dt = a.dv / 16;
        if (kn <= 1 && dt <= 2) return launch_prefill<1, 0, 2, 2>(st, a);
        if (kn <= 2 && dt <= 4) return launch_prefill<2, 0, 4, 2>(st, a);
        if (kn <= 4 && dt <= 8) return launch_prefill<4, 0, 8, 2>(st, a);
        if (kn <= 8 && dt <= 16) return launch_prefill<8, 0, 16, 1>(st, a);
    }
    if (dtype == COGS_DT_BF16 && !a.kvw && !a.absorbed && a.dn % 8 == 0 && a.dr % 8 == 0 && a.dv % 16 == 0 && a.ldq % 8 == 0 && a.q_head % 32 == 0 &&
        a.q_rot % 32 == 0 && a.q_rot >= a.dn && a.q_head - a.q_rot >= a.dr && a.ldk % 8 == 0 && a.k_head % 8 == 0 && a.ldkr % 8 == 0 &&
        a.ldv % 8 == 0 && a.v_head % 8 == 0 && a.ldo % 4 == 0 && a.o_head % 4 == 0 && g_cogs_debug.mla_rowwise == 0 &&
        a.ldk < (1 << 23) && a.ldkr < (1 << 23) && a.ldv < (1 << 23)) {       // (a tile's byte offsets are 32 bits)
        const int kn = a.q_rot / 32, kr = (a.q_head - a.q_rot) / 32, dt = a.dv / 16;
        if (kn <= 1 && kr <= 1 && dt <= 2) return launch_prefill<1, 1, 2, 2>(st, a);
        if (kn <= 2 && kr <= 1 && dt <= 4) return launch_prefill<2, 1, 4, 2>(st, a);
        if (kn <= 4 && kr <= 1 && dt <= 8) return launch_prefill<4, 1, 8, 2>(st, a);
        if (kn <= 4 && kr <= 2 && dt <= 8) return launch_prefill<4, 2, 8, 2>(st, a);
        if (kn <= 8 && kr <= 4 && dt <= 16) return launch_prefill<8, 4, 16, 1>(st, a);
    }
    if (a.dn + a.dr > RW_DIM || a.dv > 64 * RW_VREG) return COGS_E_UNSUPPORTED;
    if (dtype == COGS_DT_BF16) hipLaunchKernelGGL(mla_rowwise_kernel<bf16_t>, dim3(a.rows, a.heads), dim3(64), 0, st, a);
    else hipLaunchKernelGGL(mla_rowwise_kernel<float>, dim3(a.rows, a.heads), dim3(64), 0, st, a);
    return COGS_LAUNCH_CHECK();
}

bool cogs_k_mla_decode_fits(int kvw, int kvp) {
    return kvw % 32 == 0 && kvp % 16 == 0 && kvp <= 1024 && 48 * (kvw * 2 + 32) + 4096 <= 160 * 1024 && 32 * (kvw / 8) <= 256 * 18;
}

int cogs_k_mla_decode_splits(int nseq, int heads, int max_ctx) {
    const int keys = (int)g_cogs_debug.mla_split_keys;
    int n;
    if (keys > 0) n = (max_ctx + keys - 1) / keys;
    else {
        const int nht = (heads + 15) / 16;
        n = 512 / (nseq * nht);                           // two workgroups per CU
        const int most = (max_ctx + 63) / 64;             // shorter splits cost more in the combine than they save here
        if (n > most) n = most;
    }
    if (n < 1) n = 1;
    return n > MLA_MAX_SPLIT ? MLA_MAX_SPLIT : n;
}

// one new row per sequence: queries of kcols columns per head -> per head the weighted sum of the cache rows' value columns
int cogs_k_mla_decode(hipStream_t st, const CogsMlaDecode& a) {
    if (a.rep <= 0 || a.heads % a.rep || a.kcols % 32 || a.kcols > a.kvw || a.vcol % 16 || a.vcol + a.kvp > a.kvw || (a.bias && a.nb <= 0) ||
        a.nseq <= 0 || (long)a.nseq * (a.heads / a.rep) > 65535 || a.nsplit < 1 || a.nsplit > MLA_MAX_SPLIT || !cogs_k_mla_decode_fits(a.kvw, a.kvp) ||
        a.ldq % 8 || a.q_head % 8 || a.heads <= 0) return COGS_E_INVALID;
    MlaDecodeArgs p;
    p.Q = (const bf16_t*)a.Q; p.ldq = a.ldq; p.q_head = a.q_head; p.seqs = a.seqs; p.layer_off = a.layer_off;
    p.kvw = a.kvw; p.kcols = a.kcols; p.vcol = a.vcol; p.kvp = a.kvp; p.nsplit = a.nsplit;
    p.heads = a.heads; p.rep = a.rep; p.groups = a.heads / a.rep; p.nht = (a.rep + 15) / 16;
    p.bias = a.bias; p.nb = a.nb;
    p.part_o = a.part; p.part_ml = a.part + (size_t)a.nseq * a.nsplit * a.heads * a.kvp;
    const int dtw = (a.kvp / 16 + 3) / 4, chunks = 32 * (a.kvw / 8), nblk = a.nseq * p.groups;
    int rc;
    if (dtw <= 2 && chunks <= 256 * 4) rc = launch_decode<2, 4, 4>(st, p, nblk);
    else if (dtw <= 4 && chunks <= 256 * 6) rc = launch_decode<4, 6, 3>(st, p, nblk);
    else if (dtw <= 8 && chunks <= 256 * 10) rc = launch_decode<8, 10, 2>(st, p, nblk);
    else rc = launch_decode<16, 18, 1>(st, p, nblk);
    if (rc != COGS_OK) return rc;
    hipLaunchKernelGGL(mla_combine_kernel, dim3(a.heads, a.nseq, (a.kvp + 63) / 64), dim3(256), 0, st, p.part_o, p.part_ml, a.nsplit, a.heads,
                       a.kvp, a.sink, (bf16_t*)a.out, a.ldo, a.o_head);
    return COGS_LAUNCH_CHECK();
}
