// Gated delta rule (cogs_delta_mixer): per head a matrix S [dk][dv] carried from token to token,
//
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q.
//
// Everything here is fp32, whatever the model's dtype: the fused projection's output t, the convolution's memory, S, and all products.
//   prompts   delta_inputs (convolution, silu, unit vectors, beta, ln g) -> delta_chunk + delta_scan (32 tokens at a time on the fp32
//             matrix instructions) -> delta_out (norm and gate); delta_tail keeps the convolution's last inputs
//   decode    delta_step: one launch per layer does all of it
// A token-by-token kernel (delta_recur) serves the sizes the chunked pair has no instance for.
//
// Chunks. With G_i = sum of ln g over the chunk's tokens 0 .. i and S0 the state in front of it,
//   u_i = beta_i (v_i - e^{G_i} S0^T k_i - sum_{j<i} e^{G_i - G_j} (k_i . k_j) u_j),  i.e.  U = T diag(beta) (V - diag(e^G) K S0)
//   with T = (I + L)^-1, L_ij = beta_i e^{G_i - G_j} k_i . k_j (j < i);   O = diag(e^G) Q S0 + P U with P_ij = e^{G_i - G_j} q_i . k_j (j <= i);
//   S = e^{G_last} S0 + K^T diag(e^{G_last - G_j}) U.
// Only exponentials of differences of later minus earlier sums appear (<= 1); the sums themselves are fp64. T diag(beta), P and the
// exponentials do not depend on S: delta_chunk forms them for all chunks at once, T by forward substitution. delta_scan walks a
// sequence's chunks: a workgroup owns 16 columns of S, its four waves the 16-row tiles of S in turn.
// MFMA layout: a 16x16 accumulator holds rows 4 g + r in register r of lane group g, which is the B operand of the r-th of four
// 4-deep steps if k is taken in the order 4 g + r -- so S, R and U go from product to product in their registers, and A operands
// are 16-byte loads of four neighbouring k.
#include "common.h"
#include "kernels.h"
#include "debug.h"

namespace {

constexpr int CH = 32;                        // tokens of a chunk
constexpr int TILE = 256;                     // floats of a 16x16 tile, row-major
constexpr int REC = 6 * TILE + 3 * CH;        // per chunk and head: T beta tiles (0,0) (1,0) (1,1) | P tiles | e^G | e^{G_last - G} | e^{G_last}, ..

__device__ __forceinline__ float unit_scale(float ss) { return 1.f / sqrtf(ss + 1e-6f); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// convolution + silu of channel c at position pos; `back` input rows (stride ldt) lie in front of x, older ones in the ring
__device__ __forceinline__ float conv_silu(const CogsDelta& p, const float* x, const float* ring, int c, int pos, int back) {
    float y = p.conv[(long)(p.taps - 1) * p.channels + c] * x[c];
    for (int j = 1; j < p.taps; ++j) {
        if (j > pos) break;
        const float v = j <= back ? x[c - (long)j * p.ldt] : ring[(long)((pos - j) % p.taps) * p.channels + c];
        y = fmaf(p.conv[(long)(p.taps - 1 - j) * p.channels + c], v, y);
    }
    return y / (1.f + expf(-y));
}

// one workgroup per new row; a wave per q / k head
__global__ __launch_bounds__(256) void delta_inputs_kernel(CogsDelta p) {
    const int row = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int sq = p.rowseq[row], pos = p.rowpos[row];
    const CogsSeq s = p.seqs[sq];
    const float* x = p.t + (long)row * p.ldt;
    const float* ring = s.state + p.state_off + (long)p.heads * p.dkp * p.dvp;
    const int back = row - s.row0;
    for (int j = wid; j < 2 * p.kv_heads; j += 4) {
        float v[8], ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int d = lane + 64 * e;
            v[e] = d < p.dkp ? conv_silu(p, x, ring, j * p.dkp + d, pos, back) : 0.f;
            ss += v[e] * v[e];
        }
        float f = unit_scale(wave_sum(ss));
        if (j < p.kv_heads) f *= p.q_scale;
        float* o = (j < p.kv_heads ? p.q : p.k) + ((long)row * p.kv_heads + j % p.kv_heads) * p.dkp;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int d = lane + 64 * e;
            if (d < p.dkp) o[d] = v[e] * f;
        }
    }
    const int v0 = 2 * p.kv_heads * p.dkp, nv = p.heads * p.dvp;
    for (int i = tid; i < nv; i += 256) p.v[(long)row * nv + i] = conv_silu(p, x, ring, v0 + i, pos, back);
    const float *tb = x + v0 + 2 * nv, *ta = tb + p.headsp;
    for (int h = tid; h < p.heads; h += 256) {
        p.bg[((long)row * p.heads + h) * 2] = sigmoid_f(tb[h]);
        p.bg[((long)row * p.heads + h) * 2 + 1] = p.neg_a[h] * softplus_f(ta[h] + p.dt_bias[h]);
    }
}

// the last inputs of the convolution into the ring (behind every reader of the old ones)
__global__ __launch_bounds__(256) void delta_tail_kernel(CogsDelta p) {
    const CogsSeq s = p.seqs[blockIdx.y];
    float* ring = s.state + p.state_off + (long)p.heads * p.dkp * p.dvp;
    const int n = min(s.len, p.taps);
    for (int i = blockIdx.x * 256 + threadIdx.x; i < n * p.channels; i += gridDim.x * 256) {
        const int r = s.len - n + i / p.channels, c = i % p.channels;
        ring[(long)((s.pos0 + r) % p.taps) * p.channels + c] = p.t[(long)(s.row0 + r) * p.ldt + c];
    }
}

// token by token, a thread per column of S, S in memory
__global__ __launch_bounds__(64) void delta_recur_kernel(CogsDelta p) {
    const int h = blockIdx.y, col = blockIdx.x * 64 + threadIdx.x;
    const CogsSeq s = p.seqs[blockIdx.z];
    if (col >= p.dvp) return;
    float* S = s.state + p.state_off + (long)h * p.dkp * p.dvp + col;
    const int kh = h / (p.heads / p.kv_heads);
    for (int i = 0; i < s.len; ++i) {
        const long row = s.row0 + i;
        const bool fresh = s.pos0 + i == 0;
        const float *q = p.q + (row * p.kv_heads + kh) * p.dkp, *k = p.k + (row * p.kv_heads + kh) * p.dkp;
        const float beta = p.bg[(row * p.heads + h) * 2], g = expf(p.bg[(row * p.heads + h) * 2 + 1]);
        float a = 0.f;
        if (!fresh)
            for (int d = 0; d < p.dkp; ++d) a = fmaf(S[(long)d * p.dvp] * g, k[d], a);
        const float u = beta * (p.v[(row * p.heads + h) * p.dvp + col] - a);
        float o = 0.f;
        for (int d = 0; d < p.dkp; ++d) {
            const float v = fmaf(k[d], u, fresh ? 0.f : S[(long)d * p.dvp] * g);
            S[(long)d * p.dvp] = v;
            o = fmaf(v, q[d], o);
        }
        p.o[(row * p.heads + h) * p.dvp + col] = o;
    }
}

// A or B operands of four 4-deep steps: 16 rows (stride ld) of 16 columns
__device__ __forceinline__ f32x4 frag(const float* m, long ld, int li, int g) { return *reinterpret_cast<const f32x4*>(m + li * ld + 4 * g); }

__device__ __forceinline__ f32x4 mfma4(const f32x4& a, const f32x4& b, f32x4 c) {
#pragma unroll
    for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], c, 0, 0, 0);
    return c;
}

__device__ __forceinline__ float* chunk_rec(const CogsDelta& p, const CogsSeq& s, int seq, int chunk, int h) {
    return p.rec + ((long)(s.row0 / CH + seq + chunk) * p.heads + h) * REC;      // (a later sequence starts behind the chunks of an earlier one)
}

// what a chunk needs besides S: three waves, one per tile (0,0), (1,0), (1,1) of the 32 x 32 matrices
__global__ __launch_bounds__(192) void delta_chunk_kernel(CogsDelta p) {
    __shared__ double cum[CH];
    __shared__ float beta_s[CH];
    __shared__ __attribute__((aligned(16))) float Ls[3][16][20], Ts[3][16][20];
    const int chunk = blockIdx.x, h = blockIdx.y, seq = blockIdx.z;
    const CogsSeq s = p.seqs[seq];
    const int n = min(CH, s.len - chunk * CH);
    if (n <= 0) return;
    const int tid = threadIdx.x, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const long row0 = s.row0 + chunk * CH;
    const int kh = h / (p.heads / p.kv_heads);
    const long ld = (long)p.kv_heads * p.dkp;
    const int ta = wid > 0 ? 1 : 0, tb = wid == 2 ? 1 : 0;
    if (tid < CH) {
        const int r = min(tid, n - 1);
        const float* bg = p.bg + ((row0 + r) * p.heads + h) * 2;
        beta_s[tid] = bg[0];
        cum[tid] = tid < n ? (double)bg[1] : 0.0;
    }
    __syncthreads();
    if (tid == 0)
        for (int i = 1; i < CH; ++i) cum[i] += cum[i - 1];
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
    const long ra = min(16 * ta + li, n - 1), rb = min(16 * tb + li, n - 1);
    const float* ka = p.k + (row0 + ra) * ld + (long)kh * p.dkp + 4 * g;
    const float* qa = p.q + (row0 + ra) * ld + (long)kh * p.dkp + 4 * g;
    const float* kb = p.k + (row0 + rb) * ld + (long)kh * p.dkp + 4 * g;
    for (int d = 0; d < p.dkp; d += 16) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(ka + d), b = *reinterpret_cast<const f32x4*>(kb + d), q = *reinterpret_cast<const f32x4*>(qa + d);
        kk = mfma4(a, b, kk);
        qk = mfma4(q, b, qk);
    }
    __syncthreads();
    float* rec = chunk_rec(p, s, seq, chunk, h);
    const int j = 16 * tb + li;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int i = 16 * ta + 4 * g + r;
        const float e = j <= i ? expf((float)(cum[i] - cum[j])) : 0.f;
        const bool in = i < n && j < n;
        Ls[wid][4 * g + r][li] = in && j < i ? beta_s[i] * e * kk[r] : 0.f;
        rec[(3 + wid) * TILE + (4 * g + r) * 16 + li] = in && j <= i ? e * qk[r] : 0.f;
    }
    if (tid < CH) {
        rec[6 * TILE + tid] = expf((float)cum[tid]);
        rec[6 * TILE + CH + tid] = tid < n ? expf((float)(cum[CH - 1] - cum[tid])) : 0.f;
        if (tid == 0) rec[6 * TILE + 2 * CH] = expf((float)cum[CH - 1]);
    }
    __syncthreads();
    // inverses of the two diagonal blocks: a lane per column
    if (wid == 0 && lane < 32) {
        const int blk = lane >> 4, b = blk * 2, c = li;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float v = i == c ? 1.f : 0.f;
#pragma unroll
            for (int m = 0; m < i; ++m) v = fmaf(-Ls[b][i][m], x[m], v);
            x[i] = v;
            Ts[b][i][c] = v;
        }
    }
    __syncthreads();
    // T(1,0) = -T(1,1) L(1,0) T(0,0)
    if (wid == 0) {
        f32x4 b, m = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) b[r] = Ts[0][4 * g + r][li];
        m = mfma4(frag(&Ls[1][0][0], 20, li, g), b, m);
        f32x4 t = mfma4(frag(&Ts[2][0][0], 20, li, g), m, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
        for (int r = 0; r < 4; ++r) Ts[1][4 * g + r][li] = -t[r];
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int i = 16 * ta + 4 * g + r;
        rec[wid * TILE + (4 * g + r) * 16 + li] = i < n && j < n ? Ts[wid][4 * g + r][li] * beta_s[j] : 0.f;
    }
}

// NK: 16-row tiles of S per wave
template <int NK>
__global__ __launch_bounds__(256) void delta_scan_kernel(CogsDelta p) {
    __shared__ __attribute__((aligned(16))) f32x4 red[2][4][4][64];
    const int h = blockIdx.y, col0 = blockIdx.x * 16, seq = blockIdx.z;
    const CogsSeq s = p.seqs[seq];
    const int tid = threadIdx.x, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int kh = h / (p.heads / p.kv_heads);
    const long ld = (long)p.kv_heads * p.dkp, ldv = (long)p.heads * p.dvp;
    const float* K = p.k + s.row0 * ld + (long)kh * p.dkp;
    const float* Q = p.q + s.row0 * ld + (long)kh * p.dkp;
    const float* V = p.v + s.row0 * ldv + (long)h * p.dvp + col0 + li;
    float* O = p.o + s.row0 * ldv + (long)h * p.dvp + col0 + li;
    float* S = s.state + p.state_off + (long)h * p.dkp * p.dvp + col0 + li;
    const int tiles = p.dkp >> 4;
    f32x4 st[NK];
#pragma unroll
    for (int n = 0; n < NK; ++n) {
        st[n] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int t = wid + 4 * n;
        if (t < tiles && s.pos0 > 0)
#pragma unroll
            for (int r = 0; r < 4; ++r) st[n][r] = S[(long)(16 * t + 4 * g + r) * p.dvp];
    }
    const int nc = (s.len + CH - 1) / CH;
    for (int c = 0; c < nc; ++c) {
        const int r0 = c * CH, last = s.len - 1;
        const float* rec = chunk_rec(p, s, seq, c, h);
        f32x4 tm[3], pm[3], eg[2], ec[2];
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            tm[i] = frag(rec + i * TILE, 16, li, g);
            pm[i] = frag(rec + (3 + i) * TILE, 16, li, g);
        }
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            eg[a] = *reinterpret_cast<const f32x4*>(rec + 6 * TILE + 16 * a + 4 * g);
            ec[a] = *reinterpret_cast<const f32x4*>(rec + 6 * TILE + CH + 16 * a + 4 * g);
        }
        const float gl = rec[6 * TILE + 2 * CH];
        f32x4 v[2], x[2], y[2];
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            x[a] = y[a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int r = 0; r < 4; ++r) v[a][r] = V[(long)min(r0 + 16 * a + 4 * g + r, last) * ldv];
#pragma unroll
            for (int n = 0; n < NK; ++n) {
                const int t = wid + 4 * n;
                if (t >= tiles) continue;
                const long off = (long)min(r0 + 16 * a + li, last) * ld + 16 * t + 4 * g;
                x[a] = mfma4(*reinterpret_cast<const f32x4*>(K + off), st[n], x[a]);
                y[a] = mfma4(*reinterpret_cast<const f32x4*>(Q + off), st[n], y[a]);
            }
        }
        f32x4 (*rd)[4][64] = red[c & 1];
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            rd[wid][a][lane] = x[a];
            rd[wid][2 + a][lane] = y[a];
        }
        __syncthreads();
        f32x4 rr[2], u[2];
#pragma unroll
        for (int a = 0; a < 2; ++a) rr[a] = v[a] - eg[a] * ((rd[0][a][lane] + rd[1][a][lane]) + (rd[2][a][lane] + rd[3][a][lane]));
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        u[0] = mfma4(tm[0], rr[0], zero);
        u[1] = mfma4(tm[2], rr[1], mfma4(tm[1], rr[0], zero));
        if (wid < 2) {
            f32x4 o = eg[wid] * ((rd[0][2 + wid][lane] + rd[1][2 + wid][lane]) + (rd[2][2 + wid][lane] + rd[3][2 + wid][lane]));
            if (wid == 0) o = mfma4(pm[0], u[0], o);
            else o = mfma4(pm[2], u[1], mfma4(pm[1], u[0], o));
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = r0 + 16 * wid + 4 * g + r;
                if (i <= last) O[(long)i * ldv] = o[r];
            }
        }
#pragma unroll
        for (int a = 0; a < 2; ++a) u[a] *= ec[a];
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            const int t = wid + 4 * n;
            if (t >= tiles) continue;
            st[n] *= gl;
#pragma unroll
            for (int a = 0; a < 2; ++a) {
                f32x4 kt;
#pragma unroll
                for (int r = 0; r < 4; ++r) kt[r] = K[(long)min(r0 + 16 * a + 4 * g + r, last) * ld + 16 * t + li];
                st[n] = mfma4(kt, u[a], st[n]);
            }
        }
    }
#pragma unroll
    for (int n = 0; n < NK; ++n) {
        const int t = wid + 4 * n;
        if (t < tiles)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[(long)(16 * t + 4 * g + r) * p.dvp] = st[n][r];
    }
}

// read-outs -> the output product's operand: RMS norm over the head, weight, silu of the gate; a wave per head
template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(CogsDelta p) {
    const int row = blockIdx.x, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const long nv = (long)p.heads * p.dvp;
    const float* gate = p.t + (long)row * p.ldt + 2L * p.kv_heads * p.dkp + nv;
    for (int h = wid; h < p.heads; h += 4) {
        const float* o = p.o + row * nv + (long)h * p.dvp;
        float ss = 0.f;
        for (int d = lane * 4; d < p.dvp; d += 256) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(o + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += v[e] * v[e];
        }
        const float f = 1.f / sqrtf(wave_sum(ss) / (float)p.vdim + p.eps);
        T* y = reinterpret_cast<T*>(p.att) + (long)row * p.ldo + (long)h * p.dvp;
        for (int d = lane * 4; d < p.dvp; d += 256) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(o + d), z = *reinterpret_cast<const f32x4*>(gate + (long)h * p.dvp + d),
                        w = *reinterpret_cast<const f32x4*>(p.norm + d);
            f32x4 r;
#pragma unroll
            for (int e = 0; e < 4; ++e) r[e] = v[e] * f * w[e] * (z[e] / (1.f + expf(-z[e])));
            st4_f<T>(y + d, r);
        }
    }
}

// One new token per sequence: a workgroup per (head, sequence). S passes through registers once (NPER chunks of four columns per
// thread; 0: read twice from memory): thread = (row group, four columns), the row groups' partial sums meet in LDS.
constexpr int STEP_T = 512;
template <typename T, int NPER>
__global__ __launch_bounds__(STEP_T) void delta_step_kernel(CogsDelta p) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int row = blockIdx.y;
    const CogsSeq s = p.seqs[row];
    const int pos = s.pos0, rep = p.heads / p.kv_heads, kh = h / rep;
    const float* x = p.t + (long)row * p.ldt;
    float* S = s.state + p.state_off + (long)h * p.dkp * p.dvp;
    float* ring = s.state + p.state_off + (long)p.heads * p.dkp * p.dvp;
    const int nc = p.dvp >> 2, groups = STEP_T / nc, rg = tid / nc, c4 = tid - rg * nc;
    float *q = sm, *k = q + p.dkp, *v = k + p.dkp, *red8 = v + p.dvp, *u = red8 + 16;
    f32x4* part = reinterpret_cast<f32x4*>(u + p.dvp);             // [groups][nc]
    const bool active = rg < groups;

    f32x4 sr[NPER > 0 ? NPER : 1];
    auto load = [&](int i) {
        const int d = rg + groups * i;
        return active && d < p.dkp && pos > 0 ? *reinterpret_cast<const f32x4*>(S + (long)d * p.dvp + 4 * c4) : f32x4{0.f, 0.f, 0.f, 0.f};
    };
    if constexpr (NPER > 0) {
#pragma unroll
        for (int i = 0; i < NPER; ++i) sr[i] = load(i);
    }
    // convolution + silu of this head's q, k and v channels; the new inputs into the ring (rows other positions read stay as they are)
    const int v0 = 2 * p.kv_heads * p.dkp;
    for (int i = tid; i < 2 * p.dkp + p.dvp; i += STEP_T) {
        const int c = i < p.dkp ? kh * p.dkp + i : i < 2 * p.dkp ? (p.kv_heads + kh) * p.dkp + i - p.dkp : v0 + h * p.dvp + i - 2 * p.dkp;
        sm[i] = conv_silu(p, x, ring, c, pos, 0);
        if (i >= 2 * p.dkp || h % rep == 0) ring[(long)(pos % p.taps) * p.channels + c] = x[c];
    }
    __syncthreads();
    if (wid < 2) {
        float* z = wid ? k : q;
        float ss = 0.f;
        for (int d = lane; d < p.dkp; d += 64) ss += z[d] * z[d];
        const float f = unit_scale(wave_sum(ss)) * (wid ? 1.f : p.q_scale);
        for (int d = lane; d < p.dkp; d += 64) z[d] *= f;
    }
    const float *tb = x + v0 + 2 * p.heads * p.dvp;
    const float beta = sigmoid_f(tb[h]), g = expf(p.neg_a[h] * softplus_f(tb[p.headsp + h] + p.dt_bias[h]));
    __syncthreads();
    const int iters = NPER > 0 ? NPER : (p.dkp + groups - 1) / groups;
    f32x4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < iters; ++i) {
        const int d = rg + groups * i;
        if (active && d < p.dkp) {
            f32x4 w;
            if constexpr (NPER > 0) { sr[i] *= g; w = sr[i]; } else w = load(i) * g;
            a += w * k[d];
        }
    }
    if (active) part[rg * nc + c4] = a;
    __syncthreads();
    for (int j = tid; j < p.dvp; j += STEP_T) {
        const float* pf = reinterpret_cast<const float*>(part);
        float t = 0.f;
        for (int r = 0; r < groups; ++r) t += pf[r * p.dvp + j];
        u[j] = beta * (v[j] - t);
    }
    __syncthreads();
    const f32x4 uv = active ? *reinterpret_cast<const f32x4*>(u + 4 * c4) : f32x4{0.f, 0.f, 0.f, 0.f};
    a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < iters; ++i) {
        const int d = rg + groups * i;
        if (active && d < p.dkp) {
            f32x4 w;
            if constexpr (NPER > 0) w = sr[i]; else w = load(i) * g;
            w += uv * k[d];
            *reinterpret_cast<f32x4*>(S + (long)d * p.dvp + 4 * c4) = w;
            a += w * q[d];
        }
    }
    if (active) part[rg * nc + c4] = a;
    __syncthreads();
    // read-out, its norm and gate (v's place takes the read-out)
    float ss = 0.f;
    for (int j = tid; j < p.dvp; j += STEP_T) {
        const float* pf = reinterpret_cast<const float*>(part);
        float t = 0.f;
        for (int r = 0; r < groups; ++r) t += pf[r * p.dvp + j];
        v[j] = t;
        ss += t * t;
    }
    ss = wave_sum(ss);
    if (lane == 0) red8[wid] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < STEP_T / 64; ++w) ss += red8[w];
    const float f = 1.f / sqrtf(ss / (float)p.vdim + p.eps);
    T* y = reinterpret_cast<T*>(p.att) + (long)row * p.ldo + (long)h * p.dvp;
    const float* gate = x + v0 + (long)p.heads * p.dvp + (long)h * p.dvp;
    for (int j = tid; j < p.dvp; j += STEP_T) st_f<T>(y + j, v[j] * f * p.norm[j] * (gate[j] / (1.f + expf(-gate[j]))));
}

template <typename T>
int launch_step(hipStream_t st, const CogsDelta& p, int nseq) {
    const int nc = p.dvp / 4, groups = STEP_T / nc, nper = (p.dkp + groups - 1) / groups;
    const size_t lds = (size_t)(2 * p.dkp + 2 * p.dvp + 16) * 4 + (size_t)groups * nc * 16;
    const dim3 grid(p.heads, nseq);
#define COGS_STEP(N) hipLaunchKernelGGL((delta_step_kernel<T, N>), grid, dim3(STEP_T), lds, st, p)
    if (nper <= 2) COGS_STEP(2);
    else if (nper <= 8) COGS_STEP(8);
    else if (nper <= 32) COGS_STEP(32);
    else COGS_STEP(0);
#undef COGS_STEP
    return COGS_LAUNCH_CHECK();
}

bool sizes_ok(const CogsDelta& a) {
    return a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.taps > 0 && a.dkp % 16 == 0 && a.dvp % 16 == 0 && a.dkp <= 512 &&
           a.dvp <= 2048 && a.vdim > 0 && a.vdim <= a.dvp && a.channels == 2 * a.kv_heads * a.dkp + a.heads * a.dvp && a.ldt % 4 == 0 && a.ldo % 4 == 0;
}

}  // namespace

size_t cogs_k_delta_rec_floats(int rows, int nseq, int heads) { return (size_t)(rows / CH + nseq) * heads * REC; }

int cogs_k_delta_prompt(hipStream_t st, int dtype, const CogsDelta& a, int rows, int nseq, int max_new) {
    if (!sizes_ok(a) || rows <= 0 || nseq <= 0 || nseq > 65535 || a.heads > 65535) return COGS_E_INVALID;
    hipLaunchKernelGGL(delta_inputs_kernel, dim3(rows), dim3(256), 0, st, a);
    const int keep = (max_new < a.taps ? max_new : a.taps) * a.channels;
    hipLaunchKernelGGL(delta_tail_kernel, dim3((keep + 1023) / 1024, nseq), dim3(256), 0, st, a);
    if (a.dkp <= 256 && g_cogs_debug.delta_chunk != 0) {
        hipLaunchKernelGGL(delta_chunk_kernel, dim3((max_new + CH - 1) / CH, a.heads, nseq), dim3(192), 0, st, a);
        const dim3 grid(a.dvp / 16, a.heads, nseq);
        if (a.dkp <= 64) hipLaunchKernelGGL(delta_scan_kernel<1>, grid, dim3(256), 0, st, a);
        else if (a.dkp <= 128) hipLaunchKernelGGL(delta_scan_kernel<2>, grid, dim3(256), 0, st, a);
        else hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(256), 0, st, a);
    } else {
        hipLaunchKernelGGL(delta_recur_kernel, dim3((a.dvp + 63) / 64, a.heads, nseq), dim3(64), 0, st, a);
    }
    if (dtype == COGS_DT_BF16) hipLaunchKernelGGL(delta_out_kernel<bf16_t>, dim3(rows), dim3(256), 0, st, a);
    else hipLaunchKernelGGL(delta_out_kernel<float>, dim3(rows), dim3(256), 0, st, a);
    return COGS_LAUNCH_CHECK();
}

int cogs_k_delta_step(hipStream_t st, int dtype, const CogsDelta& a, int nseq) {
    if (!sizes_ok(a) || nseq <= 0 || nseq > 65535) return COGS_E_INVALID;
    return dtype == COGS_DT_BF16 ? launch_step<bf16_t>(st, a, nseq) : launch_step<float>(st, a, nseq);
}
