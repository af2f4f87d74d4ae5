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

// quick silu: the activation behind a short convolution
__device__ __forceinline__ float silu_q(float y) { return y * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * y)); }

// RUN consecutive rows of a sequence at a time: a wave walks one q / k head, or 64 E channels of v, or the heads' beta and ln g, with
// the convolution's window in registers and the whole run's inputs requested ahead. E: 64-channel steps of a head; TAPS: taps, rounded up
template <int E, int TAPS, int RUN>
__global__ __launch_bounds__(256) void delta_inputs_kernel(CogsDelta p) {
    const CogsSeq s = p.seqs[blockIdx.z];
    const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int i0 = blockIdx.x * RUN, n = min(RUN, s.len - i0);
    if (n <= 0) return;
    const int nqk = 2 * p.kv_heads, nv = p.heads * p.dvp, units = nqk + (nv + 64 * E - 1) / (64 * E);
    const int unit = blockIdx.y * 4 + wid, v0 = nqk * p.dkp;
    const long row0 = s.row0 + i0;
    const float* x = p.t + row0 * p.ldt;
    if (unit > units) return;
    if (unit == units) {
        const float *tb = x + v0 + 2 * nv, *ta = tb + p.headsp;
        for (int i = lane; i < n * p.heads; i += 64) {
            const int r = i / p.heads, h = i - r * p.heads;
            p.bg[(row0 * p.heads + i) * 2] = sigmoid_f(tb[(long)r * p.ldt + h]);
            p.bg[(row0 * p.heads + i) * 2 + 1] = p.neg_a[h] * softplus_f(ta[(long)r * p.ldt + h] + p.dt_bias[h]);
        }
        return;
    }
    const bool is_v = unit >= nqk;
    const int c0 = is_v ? v0 + (unit - nqk) * 64 * E : unit * p.dkp, size = is_v ? min(64 * E, v0 + nv - c0) : p.dkp;
    const float* ring = s.state + p.state_off + (long)p.heads * p.dkp * p.dvp;
    float w[TAPS][E], in[TAPS - 1 + RUN][E];          // in[TAPS - 1 + r]: row i0 + r
    int ch[E];
#pragma unroll
    for (int e = 0; e < E; ++e) ch[e] = c0 + min(lane + 64 * e, size - 1);
#pragma unroll
    for (int r = 0; r < RUN; ++r)
#pragma unroll
        for (int e = 0; e < E; ++e) in[TAPS - 1 + r][e] = x[(long)min(r, n - 1) * p.ldt + ch[e]];
#pragma unroll
    for (int j = 1; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const int i = i0 - j, pos = s.pos0 + i;
            float v = 0.f;
            if (j < p.taps && pos >= 0) v = i >= 0 ? x[ch[e] - (long)j * p.ldt] : ring[(long)(pos % p.taps) * p.channels + ch[e]];
            in[TAPS - 1 - j][e] = v;
        }
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < E; ++e) w[j][e] = j < p.taps ? p.conv[(long)(p.taps - 1 - j) * p.channels + ch[e]] : 0.f;
    float* out[E];                                    // (v's pieces may cross heads)
#pragma unroll
    for (int e = 0; e < E; ++e) {
        const int c = ch[e] - v0, hv = c / p.dvp;
        out[e] = is_v ? p.v + ((long)hv * p.rows + row0) * p.dvp + (c - hv * p.dvp)
                      : (unit < p.kv_heads ? p.q : p.k) + ((long)(unit % p.kv_heads) * p.rows + row0) * p.dkp + (ch[e] - c0);
    }
    const long ld = is_v ? p.dvp : p.dkp;
    const float scale = unit < p.kv_heads ? p.q_scale : 1.f;
#pragma unroll
    for (int r = 0; r < RUN; ++r) {
        float y[E], ss = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
            float a = w[0][e] * in[TAPS - 1 + r][e];
#pragma unroll
            for (int j = 1; j < TAPS; ++j) a = fmaf(w[j][e], in[TAPS - 1 + r - j][e], a);
            y[e] = lane + 64 * e < size ? silu_q(a) : 0.f;
            ss = fmaf(y[e], y[e], ss);
        }
        const float f = is_v ? 1.f : unit_scale(wave_sum(ss)) * scale;
#pragma unroll
        for (int e = 0; e < E; ++e)
            if (r < n && lane + 64 * e < size) out[e][r * ld] = y[e] * f;
    }
}

// the same for any size: one workgroup per new row; a wave per q / k head
__global__ __launch_bounds__(256) void delta_inputs_any_kernel(CogsDelta p) {
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
        float* o = (j < p.kv_heads ? p.q : p.k) + ((long)(j % p.kv_heads) * p.rows + row) * p.dkp;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int d = lane + 64 * e;
            if (d < p.dkp) o[d] = v[e] * f;
        }
    }
    const int v0 = 2 * p.kv_heads * p.dkp, nv = p.heads * p.dvp;
    for (int i = tid; i < nv; i += 256) p.v[((long)(i / p.dvp) * p.rows + row) * p.dvp + i % p.dvp] = conv_silu(p, x, ring, v0 + i, pos, back);
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
        const float *q = p.q + ((long)kh * p.rows + row) * p.dkp, *k = p.k + ((long)kh * p.rows + row) * p.dkp;
        const float beta = p.bg[(row * p.heads + h) * 2], g = expf(p.bg[(row * p.heads + h) * 2 + 1]);
        float a = 0.f;
        if (!fresh)
            for (int d = 0; d < p.dkp; ++d) a = fmaf(S[(long)d * p.dvp] * g, k[d], a);
        const float u = beta * (p.v[((long)h * p.rows + row) * p.dvp + col] - a);
        float o = 0.f;
        for (int d = 0; d < p.dkp; ++d) {
            const float v = fmaf(k[d], u, fresh ? 0.f : S[(long)d * p.dvp] * g);
            S[(long)d * p.dvp] = v;
            o = fmaf(v, q[d], o);
        }
        p.o[((long)h * p.rows + row) * p.dvp + col] = o;
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
    const long k0 = ((long)kh * p.rows + row0) * p.dkp + 4 * g;
    const int ta = wid > 0 ? 1 : 0, tb = wid == 2 ? 1 : 0;
    if (tid < CH) {
        const int r = min(tid, n - 1);
        const float* bg = p.bg + ((row0 + r) * p.heads + h) * 2;
        beta_s[tid] = bg[0];
        double sum = tid < n ? (double)bg[1] : 0.0;
#pragma unroll
        for (int o = 1; o < CH; o *= 2) {
            const double before = __shfl_up(sum, o, CH);
            if (tid >= o) sum += before;
        }
        cum[tid] = sum;
    }
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
    const long ra = min(16 * ta + li, n - 1), rb = min(16 * tb + li, n - 1);
    const float* ka = p.k + k0 + ra * p.dkp;
    const float* qa = p.q + k0 + ra * p.dkp;
    const float* kb = p.k + k0 + rb * p.dkp;
    for (int d = 0; d < p.dkp; d += 64) {              // four 16-wide steps in flight; steps past the end are not multiplied
        f32x4 a[4], b[4], q[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int o = min(d + 16 * e, p.dkp - 16);
            a[e] = *reinterpret_cast<const f32x4*>(ka + o);
            b[e] = *reinterpret_cast<const f32x4*>(kb + o);
            q[e] = *reinterpret_cast<const f32x4*>(qa + o);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            if (d + 16 * e >= p.dkp) break;
            kk = mfma4(a[e], b[e], kk);
            qk = mfma4(q[e], b[e], qk);
        }
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

// what a wave needs of one chunk; loaded one chunk ahead
template <int NK>
struct ScanIn {
    f32x4 tm[3], pm[2], eg[2], ec[2], v[2], k[2][NK], q[2][NK], kt[2][NK];
    float gl;
};

// NK: 16-row tiles of S per wave. A chunk: S^T k from the state (partial sums of the waves meet in LDS: one barrier), then, while they
// do, S^T q; U; the new state beside P U. The read-outs' partial sums ride on the next chunk's barrier, and waves 0 and 1 finish and
// store 16 rows of them each behind it (waves 2 and 3 form copies of P U that nobody reads: they would wait otherwise). One wave per
// SIMD issues in order, so the next chunk's loads are spread between the matrix instructions, and no product is one long chain.
template <int NK>
__global__ __launch_bounds__(256, 1) void delta_scan_kernel(CogsDelta p) {
    __shared__ __attribute__((aligned(16))) f32x4 red[2][4][4][64];
    // workgroups go round the XCDs: the columns of a head stay on one, whose L2 then serves its K and Q once
    const int ng = p.dvp >> 4, place = blockIdx.x >> 3, h = (blockIdx.x & 7) + 8 * (place / ng), col0 = (place % ng) * 16, seq = blockIdx.z;
    if (h >= p.heads) return;
    const CogsSeq s = p.seqs[seq];
    const int tid = threadIdx.x, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(tid >> 6), half = wid & 1;
    const int kh = h / (p.heads / p.kv_heads);
    const int ld = p.dkp, ldv = p.dvp;
    const float* K = p.k + ((long)kh * p.rows + s.row0) * ld;
    const float* Q = p.q + ((long)kh * p.rows + s.row0) * ld;
    const float* V = p.v + ((long)h * p.rows + s.row0) * ldv + col0;
    float* O = p.o + ((long)h * p.rows + s.row0) * ldv + col0;
    float* S = s.state + p.state_off + (long)h * p.dkp * p.dvp + col0 + li;
    const int tiles = p.dkp >> 4;
    f32x4 st[NK];
    int tn[NK];                                  // tiles past the end repeat the last one, and their S is kept at zero
    float live[NK];
#pragma unroll
    for (int n = 0; n < NK; ++n) {
        st[n] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int t = wid + 4 * n;
        tn[n] = 16 * min(t, tiles - 1);
        live[n] = t < tiles ? 1.f : 0.f;
        if (t < tiles && s.pos0 > 0)
#pragma unroll
            for (int r = 0; r < 4; ++r) st[n][r] = S[(long)(16 * t + 4 * g + r) * p.dvp];
    }
    const int nc = (s.len + CH - 1) / CH;
    // a lane's places in a chunk's rows (bytes); a ragged last chunk repeats its last row
    unsigned ko[2], to[2][4], vo[2][4], oo[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) oo[r] = ((16 * half + 4 * g + r) * ldv + li) * 4;
    const unsigned ro = (li * 16 + 4 * g) * 4, ego = 16 * g;
    auto places = [&](int valid) {
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            ko[a] = (min(16 * a + li, valid - 1) * ld + 4 * g) * 4;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = min(16 * a + 4 * g + r, valid - 1);
                to[a][r] = (row * ld + li) * 4;
                vo[a][r] = (row * ldv + li) * 4;
            }
        }
    };
    places(CH);
    auto at4 = [](const float* base, unsigned bytes) { return *reinterpret_cast<const f32x4*>(reinterpret_cast<const char*>(base) + bytes); };
    auto at1 = [](const float* base, unsigned bytes) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + bytes); };
    // load i of a chunk: the 12 NK + 18 of them in the order of their use
    struct From { const float *k, *q, *v, *rec; };
    From f{K, Q, V, chunk_rec(p, s, seq, 0, h)};
    const long step_k = (long)CH * ld, step_v = (long)CH * ldv, step_rec = (long)p.heads * REC;
    int at = 0;                                                // the chunk f points to
    auto advance = [&] {                                       // (the last chunk is loaded again rather than nothing)
        if (at + 1 >= nc) return;
        ++at;
        f.k += step_k; f.q += step_k; f.v += step_v; f.rec += step_rec;
        if ((at + 1) * CH > s.len) places(s.len - at * CH);
    };
    constexpr int L_K = 2 * NK, L_V = L_K + 8, L_TM = L_V + 3, L_EG = L_TM + 2, L_Q = L_EG + 2 * NK, L_EC = L_Q + 2, L_KT = L_EC + 8 * NK, L_ALL = L_KT + 3;
    auto load = [&](ScanIn<NK>& in, int i) {
        if (i < L_K) in.k[i & 1][i >> 1] = at4(f.k + tn[i >> 1], ko[i & 1]);
        else if (i < L_V) in.v[(i - L_K) >> 2][(i - L_K) & 3] = at1(f.v, vo[(i - L_K) >> 2][(i - L_K) & 3]);
        else if (i < L_TM) in.tm[i - L_V] = at4(f.rec + (i - L_V) * TILE, ro);
        else if (i < L_EG) in.eg[i - L_TM] = at4(f.rec + 6 * TILE + 16 * (i - L_TM), ego);
        else if (i < L_Q) in.q[(i - L_EG) & 1][(i - L_EG) >> 1] = at4(f.q + tn[(i - L_EG) >> 1], ko[(i - L_EG) & 1]);
        else if (i < L_EC) in.ec[i - L_Q] = at4(f.rec + 6 * TILE + CH + 16 * (i - L_Q), ego);
        else if (i < L_KT) in.kt[((i - L_EC) >> 2) & 1][(i - L_EC) >> 3][(i - L_EC) & 3] = at1(f.k + tn[(i - L_EC) >> 3], to[((i - L_EC) >> 2) & 1][(i - L_EC) & 3]);
        else if (i < L_ALL - 1) in.pm[i - L_KT] = at4(f.rec + (3 + half + (i - L_KT)) * TILE, ro);      // half 0: P(0,0) and one without use; 1: P(1,0), P(1,1)
        else if (i < L_ALL) in.gl = f.rec[6 * TILE + 2 * CH];
    };
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const float second = half ? 1.f : 0.f;                     // rows 0 .. 15 have no P(0,1)
    f32x4 y[2] = {zero, zero}, po = zero, peg = zero;          // the previous chunk's: partial S^T q, P U and e^G of this wave's rows
    auto sum4 = [&](f32x4 (*rd)[4][64], int a) { return (rd[0][a][lane] + rd[1][a][lane]) + (rd[2][a][lane] + rd[3][a][lane]); };
    auto store = [&](int c, const f32x4& o, bool ragged) {
        float* oc = O + (long)c * CH * ldv;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (!ragged || c * CH + 16 * half + 4 * g + r < s.len) *reinterpret_cast<float*>(reinterpret_cast<char*>(oc) + oo[r]) = o[r];
    };
    auto meet = [&] {                                          // (loads of the next chunk stay in flight)
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
    };
    auto mfma = [](float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); };
    // chunk c from `in`, the next one into nx
    auto chunk = [&](int c, const ScanIn<NK>& in, ScanIn<NK>& nx) {
        advance();
        constexpr int STEPS = 8 * NK + 8 * NK / 2 + 6;         // pairs of matrix instructions
        int step = 0, done = 0;
        auto feed = [&] {                                      // this pair's share of the loads
            ++step;
#pragma unroll
            for (int i = 0; i < L_ALL; ++i)
                if (i >= done && i < (L_ALL * step + STEPS - 1) / STEPS) load(nx, i);
            done = (L_ALL * step + STEPS - 1) / STEPS;
            __builtin_amdgcn_sched_barrier(0);
        };
        f32x4 x[2][2] = {{zero, zero}, {zero, zero}};          // [16 rows][half of the depth]
#pragma unroll
        for (int n = 0; n < NK; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
#pragma unroll
                for (int a = 0; a < 2; ++a) x[a][r & 1] = mfma(in.k[a][n][r], st[n][r], x[a][r & 1]);
                feed();
            }
        f32x4 (*rd)[4][64] = red[c & 1];
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            rd[wid][2 + a][lane] = y[a];
            rd[wid][a][lane] = x[a][0] + x[a][1];
        }
        meet();
        f32x4 part[3][4];
#pragma unroll
        for (int a = 0; a < 3; ++a)
#pragma unroll
            for (int w = 0; w < 4; ++w) part[a][w] = rd[w][a < 2 ? a : 2 + half][lane];
        __builtin_amdgcn_sched_barrier(0);
        y[0] = y[1] = zero;
        f32x4 y2[2] = {zero, zero};
#pragma unroll
        for (int n = 0; n < NK; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
#pragma unroll
                for (int a = 0; a < 2; ++a) {
                    f32x4& t = (r & 1) ? y2[a] : y[a];
                    t = mfma(in.q[a][n][r], st[n][r], t);
                }
                feed();
            }
        f32x4 rr[2], u[2] = {zero, zero}, u1 = zero;
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            rr[a] = in.v[a] - in.eg[a] * ((part[a][0] + part[a][1]) + (part[a][2] + part[a][3]));
            y[a] += y2[a];
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {                          // three chains
            u[0] = mfma(in.tm[0][r], rr[0][r], u[0]);
            u[1] = mfma(in.tm[1][r], rr[0][r], u[1]);
            if (r & 1) feed();
            u1 = mfma(in.tm[2][r], rr[1][r], u1);
            feed();
        }
        u[1] += u1;
        const f32x4 o = po + peg * ((part[2][0] + part[2][1]) + (part[2][2] + part[2][3]));
        f32x4 ue[2], pa = zero, pb = zero, s2[NK];
        const f32x4 up = u[1] * second;
#pragma unroll
        for (int a = 0; a < 2; ++a) ue[a] = u[a] * in.ec[a];
#pragma unroll
        for (int n = 0; n < NK; ++n) {
            st[n] *= in.gl;
            s2[n] = zero;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
#pragma unroll
            for (int n = 0; n < NK; ++n) {
                st[n] = mfma(in.kt[0][n][r], ue[0][r], st[n]);
                s2[n] = mfma(in.kt[1][n][r], ue[1][r], s2[n]);
                feed();
            }
            pa = mfma(in.pm[0][r], u[0][r], pa);
            pb = mfma(in.pm[1][r], up[r], pb);
        }
#pragma unroll
        for (int n = 0; n < NK; ++n) st[n] = (st[n] + s2[n]) * live[n];
        po = pa + pb;
        peg = half ? in.eg[1] : in.eg[0];
        if (c > 0 && wid < 2) store(c - 1, o, false);
    };
    ScanIn<NK> in0, in1;
    if (s.len < CH) places(s.len);
#pragma unroll
    for (int i = 0; i < L_ALL; ++i) load(in0, i);
    for (int c = 0; c < nc; c += 2) {
        chunk(c, in0, in1);
        if (c + 1 >= nc) break;
        chunk(c + 1, in1, in0);
    }
    {
        f32x4 (*rd)[4][64] = red[nc & 1];
#pragma unroll
        for (int a = 0; a < 2; ++a) rd[wid][2 + a][lane] = y[a];
        meet();
        if (wid < 2) store(nc - 1, po + peg * sum4(rd, 2 + half), true);
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
        const float* o = p.o + ((long)h * p.rows + row) * p.dvp;
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

void launch_inputs(hipStream_t st, const CogsDelta& a, int rows, int nseq, int max_new) {
    const int nv = a.heads * a.dvp;
    const auto grid = [&](int e, int run) { return dim3((max_new + run - 1) / run, (2 * a.kv_heads + (nv + 64 * e - 1) / (64 * e) + 1 + 3) / 4, nseq); };
    if (a.taps <= 4 && a.dkp <= 64) hipLaunchKernelGGL((delta_inputs_kernel<1, 4, 16>), grid(1, 16), dim3(256), 0, st, a);
    else if (a.taps <= 4 && a.dkp <= 128) hipLaunchKernelGGL((delta_inputs_kernel<2, 4, 16>), grid(2, 16), dim3(256), 0, st, a);
    else if (a.taps <= 8 && a.dkp <= 256) hipLaunchKernelGGL((delta_inputs_kernel<4, 8, 8>), grid(4, 8), dim3(256), 0, st, a);
    else hipLaunchKernelGGL(delta_inputs_any_kernel, dim3(rows), dim3(256), 0, st, a);
}

bool sizes_ok(const CogsDelta& a) {
    return a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.taps > 0 && a.dkp % 16 == 0 && a.dvp % 16 == 0 && a.dkp <= 512 &&
           a.dvp <= 2048 && a.vdim > 0 && a.vdim <= a.dvp && a.channels == 2 * a.kv_heads * a.dkp + a.heads * a.dvp && a.ldt % 4 == 0 && a.ldo % 4 == 0;
}

}  // namespace

size_t cogs_k_delta_rec_floats(int rows, int nseq, int heads) { return (size_t)(rows / CH + nseq) * heads * REC; }

int cogs_k_delta_prompt(hipStream_t st, int dtype, const CogsDelta& a, int rows, int nseq, int max_new) {
    if (!sizes_ok(a) || rows <= 0 || nseq <= 0 || nseq > 65535 || a.heads > 65535) return COGS_E_INVALID;
    launch_inputs(st, a, rows, nseq, max_new);
    const int keep = (max_new < a.taps ? max_new : a.taps) * a.channels;
    hipLaunchKernelGGL(delta_tail_kernel, dim3((keep + 1023) / 1024, nseq), dim3(256), 0, st, a);
    if (a.dkp <= 256 && g_cogs_debug.delta_chunk != 0) {
        hipLaunchKernelGGL(delta_chunk_kernel, dim3((max_new + CH - 1) / CH, a.heads, nseq), dim3(192), 0, st, a);
        const dim3 grid((a.heads + 7) / 8 * 8 * (a.dvp / 16), 1, nseq);
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
