// Decoder-only models described layer by layer (include/cogs.h, cogs_decoder_*): the launch sequence of one step of a batch of
// sequences. A mechanism is a function over one layer's descriptor; what a model is made of is data.
#include "ctx.h"
#include "debug.h"

#include <math.h>
#include <new>

namespace {

inline int up(int v, int m) { return (v + m - 1) / m * m; }
inline void mx(int& a, int b) { a = b > a ? b : a; }
inline void mx(long& a, long b) { a = b > a ? b : a; }

// padded sizes and places of one layer's mixer (include/cogs.h has the rules)
struct LatentGeom {
    int qrp, kvp, rotc, kvw, dn, dr, dq, dk, dv, oin, headsp, ldt, kvcols;
    bool own;
    int src;              // layer whose cache rows are read
    int rope;             // rotation table
};
struct AttnGeom { int dk, dv, kvw, ldt, oin; };
struct DeltaGeom { int dk, dv, headsp, channels, ldt, oin; };
struct Geom {
    LatentGeom lat; AttnGeom att; DeltaGeom del;
    int rows_width;       // columns this layer adds to a token's cache row
    long state;           // floats it adds to a sequence's state
};
// one pass through a layer: where its cache rows (first column) and its state (first float) lie
struct Run { int layer; long cache_off, state_off; };

}  // namespace

struct CogsDecoder {
    cogs_decoder_weights w{};
    std::vector<cogs_decoder_layer> layers;
    std::vector<Geom> geom;
    std::vector<Run> runs;
    std::vector<CogsRopeSet> sets;
    CogsRopeSet* sets_dev = nullptr;
    double* freq_dev = nullptr;
    int wp = 0, vocabp = 0, max_pairs = 0;
    long rope_width = 0, cache_width = 0;     // floats per row of all rotation tables; elements per token of a cache
    long state_floats = 0;                    // fp32 recurrent state of a sequence
    // largest row widths over the layers
    int max_t32 = 0, max_cq = 0, max_q = 0, max_o = 0, max_ff = 0, max_kvcols = 0, max_kvw = 0, max_heads = 0;
    long max_qlat = 0, max_olat = 0;
    int max_dqk = 0, max_dv = 0, max_dheads = 0;       // gated delta rule: kv_heads x dim, heads x vdim, heads
    bool att_tail = false;
};

void cogs_decoder_free(CogsDecoder* d) {
    if (!d) return;
    if (d->sets_dev) (void)hipFree(d->sets_dev);
    if (d->freq_dev) (void)hipFree(d->freq_dev);
    delete d;
}

namespace {

struct Work {
    float* x; void *h, *y, *cq, *q, *att, *act, *hn, *ctx, *kvx, *qlat, *olat;
    float *t32, *gate, *rope, *part, *dq, *dk, *dv, *dbg, *dout, *drec;
    CogsSeq* seqs; int *rowseq, *rowpos, *want;
    size_t bytes;
};

// sequences of one token each: absorbed attention, key-split attention (mla.hip), one-launch delta rule (delta.hip)
inline bool token_step(int rows, int nseq) { return rows == nseq; }
inline bool absorbed_step(int rows, int nseq) { return token_step(rows, nseq) && g_cogs_debug.mla_absorb != 0; }

Work carve(const CogsDecoder& d, int S, int nseq, int64_t C, int n_want, void* ws, size_t cap) {
    Carver c(ws, cap);
    const size_t es = esize(d.w.dtype), n = (size_t)S;
    Work k{};
    k.x = (float*)c.take(n * d.wp * 4 * (d.w.streams > 0 ? d.w.streams : 1));
    k.h = c.take(n * d.wp * es);
    k.y = c.take(n * d.wp * es);
    k.t32 = (float*)c.take(n * d.max_t32 * 4);
    k.cq = c.take(n * d.max_cq * es);
    k.q = c.take(n * d.max_q * es);
    k.att = c.take(n * d.max_o * es);
    k.act = c.take(n * d.max_ff * es);
    k.gate = (float*)c.take(n * d.max_heads * 4);
    k.rope = (float*)c.take(n * d.rope_width * 4);
    k.hn = c.take((size_t)n_want * d.wp * es);
    k.seqs = (CogsSeq*)c.take(nseq * sizeof(CogsSeq));
    k.rowseq = (int*)c.take(n * 4);
    k.rowpos = (int*)c.take(n * 4);
    k.want = (int*)c.take((size_t)n_want * 4);
    if (token_step(S, nseq)) {
        size_t part = 0;
        for (size_t l = 0; l < d.geom.size(); ++l) {
            size_t b = 0;
            if (d.layers[l].mixer == COGS_MIX_LATENT && absorbed_step(S, nseq)) {
                const int heads = d.layers[l].latent.heads;
                b = (size_t)nseq * cogs_k_mla_decode_splits(nseq, heads, (int)C) * heads * (d.geom[l].lat.kvp + 2) * 4;
            } else if (d.layers[l].mixer == COGS_MIX_ATTENTION) {
                const cogs_attn_mixer& m = d.layers[l].attn;
                b = (size_t)nseq * cogs_k_mla_decode_splits(nseq * m.kv_heads, m.heads / m.kv_heads, (int)C) * m.heads * (d.geom[l].att.dv + 2) * 4;
            }
            part = b > part ? b : part;
        }
        k.part = (float*)c.take(part);
    }
    if (absorbed_step(S, nseq)) {
        k.qlat = c.take(n * d.max_qlat * es);
        k.olat = c.take(n * d.max_olat * es);
    } else {
        k.kvx = c.take((size_t)C * d.max_kvcols * es);
        if (nseq > 1) k.ctx = c.take((size_t)C * d.max_kvw * es);
    }
    if (!token_step(S, nseq) && d.max_dheads > 0) {
        k.dq = (float*)c.take(n * d.max_dqk * 4);
        k.dk = (float*)c.take(n * d.max_dqk * 4);
        k.dv = (float*)c.take(n * d.max_dv * 4);
        k.dout = (float*)c.take(n * d.max_dv * 4);
        k.dbg = (float*)c.take(n * d.max_dheads * 2 * 4);
        k.drec = (float*)c.take(cogs_k_delta_rec_floats(S, nseq, d.max_dheads) * 4);
    }
    k.bytes = c.off;
    return k;
}

struct Step {
    cogs_handle h; hipStream_t st; const CogsDecoder& d; Work k;
    const std::vector<CogsSeq>& seqs;
    int S, nseq, max_new, max_ctx; int64_t C;

    const void* at(const void* p, size_t elems) const { return (const char*)p + elems * esize(d.w.dtype); }

    // C[rows, N] = A . W^T with an epilogue: few rows stream the weights, one row takes the GEMV, the rest the tiled kernels
    int lin(CogsGemm& g) {
        PROF(COGS_PROF_GEMM);
        g.dtype = d.w.dtype;
        if (g_cogs_debug.gemm_skinny != 0 && cogs_k_gemm_skinny_fits(g)) return cogs_k_gemm_skinny(st, g);
        if (g.K < 128) g.force_small_tile = 1;      // the deep-pipelined kernels want at least two 64-wide slabs
        return cogs_k_gemm(st, g);
    }

    int latent_attention(const Run& run) {
        const cogs_latent_mixer& m = d.layers[run.layer].latent;
        const LatentGeom& G = d.geom[run.layer].lat;
        const CogsRopeSet& R = d.sets[G.rope];
        const int dt = d.w.dtype;
        {   // query latent | kv latent | rotated key part | gate logits
            CogsGemm g;
            g.A = k.h; g.lda = d.wp; g.W = m.in_w; g.ldw = d.wp; g.C = k.t32; g.ldc = G.ldt; g.M = S; g.N = G.ldt; g.K = d.wp; g.out_f32 = 1;
            COGS_TRY(lin(g));
        }
        {
            CogsMlaLatent a{};
            a.t = k.t32; a.ldt = G.ldt; a.qr = m.q_rank; a.qrp = G.qrp; a.kvr = m.kv_rank; a.kvp = G.kvp; a.dr = m.rot_dim; a.krc = G.rotc;
            a.own_kv = G.own; a.gate_col = m.gated ? G.qrp + (G.own ? G.kvw : 0) : -1; a.heads = m.heads;
            a.q_norm = m.q_norm; a.kv_norm = m.kv_norm; a.eps = d.w.eps;
            a.rope = k.rope + R.off * S; a.rope_pairs = R.pairs; a.rope_first = R.first;
            a.cq = k.cq; a.gate = k.gate; a.seqs = k.seqs; a.rowseq = k.rowseq; a.rowpos = k.rowpos; a.layer_off = run.cache_off;
            PROF(COGS_PROF_NORM);
            COGS_TRY(cogs_k_mla_latent(st, dt, a, S));
        }
        const int qcols = m.heads * G.dq;
        {   // rotated queries in log2 score units
            CogsGemm g;
            g.A = k.cq; g.lda = G.qrp; g.W = m.q_w; g.ldw = G.qrp; g.C = k.q; g.ldc = qcols; g.M = S; g.N = qcols; g.K = G.qrp;
            g.rope_cos = k.rope + R.off * S; g.rope_cols = qcols; g.head_dim = G.dq;
            g.q_scale = m.scale * 1.4426950408889634f; g.q_cols = qcols;
            COGS_TRY(lin(g));
        }
        const float* gate = m.gated ? k.gate : nullptr;
        if (absorbed_step(S, nseq)) {
            {
                CogsHeadGemm a{k.q, qcols, G.dq, m.k_abs, k.qlat, (long)m.heads * G.kvw, G.kvw, S, m.heads, G.kvp, G.dk, nullptr, G.rotc, G.dk, G.dr};
                PROF(COGS_PROF_GEMM);
                COGS_TRY(cogs_k_head_gemm(st, dt, a));
            }
            if (dt == COGS_DT_BF16 && g_cogs_debug.mla_rowwise == 0 && cogs_k_mla_decode_fits(G.kvw, G.kvp)) {
                CogsMlaDecode a{k.qlat, (long)m.heads * G.kvw, G.kvw, k.seqs, nseq, run.cache_off, G.kvw, G.kvw, 0, G.kvp, m.heads, m.heads,
                                cogs_k_mla_decode_splits(nseq, m.heads, max_ctx), m.sink, k.part, k.olat, (long)m.heads * G.kvp, G.kvp, nullptr, 0};
                PROF(COGS_PROF_ATTN);
                COGS_TRY(cogs_k_mla_decode(st, a));
            } else {
                CogsMla a{};
                a.Q = k.qlat; a.ldq = (long)m.heads * G.kvw; a.q_head = G.kvw; a.q_rot = G.kvp; a.ldk = a.ldkr = a.ldv = G.kvw;
                a.O = k.olat; a.ldo = (long)m.heads * G.kvp; a.o_head = G.kvp; a.dn = G.kvp; a.dr = G.rotc; a.dv = G.kvp; a.heads = m.heads;
                a.sink = m.sink; a.seqs = k.seqs; a.nseq = nseq; a.rowseq = k.rowseq; a.rows = S; a.max_new = 1;
                a.absorbed = 1; a.layer_off = run.cache_off; a.kr_col = G.kvp;
                PROF(COGS_PROF_ATTN);
                COGS_TRY(cogs_k_mla_attention(st, dt, a));
            }
            CogsHeadGemm a{k.olat, (long)m.heads * G.kvp, G.kvp, at(m.kv_w, (size_t)m.heads * G.dn * G.kvp), k.att, G.oin, G.dv, S, m.heads,
                           G.dv, G.kvp, gate, 0, 0, 0};
            PROF(COGS_PROF_GEMM);
            COGS_TRY(cogs_k_head_gemm(st, dt, a));
        } else {
            const void* ctx = k.ctx;
            if (nseq == 1) ctx = at(seqs[0].cache, (size_t)run.cache_off * seqs[0].max_len);
            else { PROF(COGS_PROF_OTHER); COGS_TRY(cogs_k_mla_gather(st, dt, k.seqs, nseq, max_ctx, run.cache_off, G.kvw, k.ctx)); }
            {   // every head's keys and values of the whole context
                CogsGemm g;
                g.A = ctx; g.lda = G.kvw; g.W = m.kv_w; g.ldw = G.kvp; g.C = k.kvx; g.ldc = G.kvcols; g.M = (int)C; g.N = G.kvcols; g.K = G.kvp;
                COGS_TRY(lin(g));
            }
            CogsMla a{};
            a.Q = k.q; a.ldq = qcols; a.q_head = G.dq; a.q_rot = G.dk; a.K = k.kvx; a.ldk = G.kvcols; a.k_head = G.dn;
            a.KR = at(ctx, G.kvp); a.ldkr = G.kvw; a.V = at(k.kvx, (size_t)m.heads * G.dn); a.ldv = G.kvcols; a.v_head = G.dv;
            a.O = k.att; a.ldo = G.oin; a.o_head = G.dv; a.dn = G.dn; a.dr = G.dr; a.dv = G.dv; a.heads = m.heads;
            a.sink = m.sink; a.gate = gate; a.seqs = k.seqs; a.nseq = nseq; a.rowseq = k.rowseq; a.rows = S; a.max_new = max_new;
            PROF(COGS_PROF_ATTN);
            COGS_TRY(cogs_k_mla_attention(st, dt, a));
        }
        return project(m.o_w, G.oin);
    }

    // attention rows -> sublayer output
    int project(const void* o_w, int oin) {
        CogsGemm g;
        g.A = k.att; g.lda = oin; g.W = o_w; g.ldw = oin; g.C = k.y; g.ldc = d.wp; g.M = S; g.N = d.wp; g.K = oin;
        return lin(g);
    }

    int attention(const Run& run) {
        const cogs_attn_mixer& m = d.layers[run.layer].attn;
        const AttnGeom& G = d.geom[run.layer].att;
        const int dt = d.w.dtype, rep = m.heads / m.kv_heads;
        {
            CogsGemm g;
            g.A = k.h; g.lda = d.wp; g.W = m.in_w; g.ldw = d.wp; g.C = k.t32; g.ldc = G.ldt; g.M = S; g.N = G.ldt; g.K = d.wp; g.out_f32 = 1;
            COGS_TRY(lin(g));
        }
        {
            CogsAttnHeads a{k.t32, G.ldt, m.heads, m.kv_heads, m.dim, G.dk, G.dv, G.kvw, m.qk_norm, d.w.eps, m.scale, m.temp_coef, m.temp_every,
                            k.q, k.seqs, k.rowseq, k.rowpos, run.cache_off};
            PROF(COGS_PROF_NORM);
            COGS_TRY(cogs_k_attn_heads(st, dt, a, S));
        }
        if (token_step(S, nseq) && dt == COGS_DT_BF16 && g_cogs_debug.mla_rowwise == 0 && cogs_k_mla_decode_fits(G.kvw, G.dv)) {
            CogsMlaDecode a{k.q, (long)m.heads * G.dk, G.dk, k.seqs, nseq, run.cache_off, G.kvw, G.dk, G.dk, G.dv, m.heads, rep,
                            cogs_k_mla_decode_splits(nseq * m.kv_heads, rep, max_ctx), nullptr, k.part, k.att, G.oin, G.dv, m.dist_bias, m.dist_n};
            PROF(COGS_PROF_ATTN);
            COGS_TRY(cogs_k_mla_decode(st, a));
        } else {
            CogsMla a{};
            a.Q = k.q; a.ldq = (long)m.heads * G.dk; a.q_head = a.q_rot = G.dk; a.ldk = a.ldv = G.kvw; a.O = k.att; a.ldo = G.oin; a.o_head = G.dv;
            a.dn = G.dk; a.dv = G.dv; a.heads = m.heads; a.seqs = k.seqs; a.nseq = nseq; a.rowseq = k.rowseq; a.rows = S; a.max_new = max_new;
            a.layer_off = run.cache_off; a.kvw = G.kvw; a.v_col = G.dk; a.rep = rep; a.bias = m.dist_bias; a.nb = m.dist_n;
            PROF(COGS_PROF_ATTN);
            COGS_TRY(cogs_k_mla_attention(st, dt, a));
        }
        return project(m.o_w, G.oin);
    }

    int delta(const Run& run) {
        const cogs_delta_mixer& m = d.layers[run.layer].delta;
        const DeltaGeom& G = d.geom[run.layer].del;
        {
            CogsGemm g;
            g.A = k.h; g.lda = d.wp; g.W = m.in_w; g.ldw = d.wp; g.C = k.t32; g.ldc = G.ldt; g.M = S; g.N = G.ldt; g.K = d.wp; g.out_f32 = 1;
            COGS_TRY(lin(g));
        }
        CogsDelta a{k.t32, G.ldt, m.heads, G.headsp, m.kv_heads, G.dk, G.dv, m.vdim, m.taps, G.channels, m.conv, m.neg_a, m.dt_bias, m.norm, d.w.eps,
                    1.f / sqrtf((float)m.dim), S, k.dq, k.dk, k.dv, k.dbg, k.dout, k.drec, k.att, G.oin, k.seqs, k.rowseq, k.rowpos, run.state_off};
        {
            PROF(COGS_PROF_ATTN);
            if (token_step(S, nseq)) COGS_TRY(cogs_k_delta_step(st, d.w.dtype, a, nseq));
            else COGS_TRY(cogs_k_delta_prompt(st, d.w.dtype, a, S, nseq, max_new));
        }
        return project(m.o_w, G.oin);
    }

    int mixer(const Run& run) {
        // columns of k.att past a layer's heads are read by its output product (times zero weights): they must hold numbers
        switch (d.layers[run.layer].mixer) {
            case COGS_MIX_ATTENTION: return attention(run);
            case COGS_MIX_DELTA: return delta(run);
            default: return latent_attention(run);
        }
    }

    int mlp(int l) {
        const cogs_decoder_mlp& m = d.layers[l].mlp;
        const int ffp = up(m.ff, 64);
        CogsGemm g;
        g.A = k.h; g.lda = d.wp; g.W = m.up_w; g.ldw = d.wp; g.C = k.act; g.ldc = ffp; g.bias = m.up_b; g.M = S;
        g.N = m.act == COGS_ACT_SWIGLU ? 2 * ffp : ffp; g.K = d.wp; g.act = m.act;
        COGS_TRY(lin(g));
        CogsGemm g2;
        g2.A = k.act; g2.lda = ffp; g2.W = m.down_w; g2.ldw = ffp; g2.C = k.y; g2.ldc = d.wp; g2.bias = m.down_b; g2.M = S; g2.N = d.wp; g2.K = ffp;
        return lin(g2);
    }

    // x from the embeddings, or x += norm(y) through the sublayer's (`from`) hyper-connections; then h = norm of what `to` reads
    int stream(const void* embeds, const float* y_gamma, const cogs_hyper* from, const cogs_hyper* to, const float* out_gamma, float* sum) {
        CogsStreamNorm a;
        a.x = k.x; a.embeds = embeds; a.y = embeds ? nullptr : k.y; a.y_gamma = y_gamma; a.out = out_gamma ? k.h : nullptr; a.out_gamma = out_gamma;
        a.rows = S; a.H = d.w.width; a.Hp = d.wp; a.eps = d.w.eps;
        if (embeds) { a.embed_scale = d.w.embed_scale; a.pos = d.w.pos; a.rowpos = k.rowpos; }
        a.streams = d.w.streams; a.sum = sum;
        if (d.w.streams > 0) {
            if (from) { a.mix = from->mix; a.out_w = from->out; }
            if (to) a.in_w = to->in;
        }
        PROF(COGS_PROF_NORM);
        return cogs_k_stream_norm(st, d.w.dtype, a);
    }
};

}  // namespace

extern "C" {

cogs_status cogs_decoder_load(cogs_handle h, const cogs_decoder_weights* w) {
    if (!h || !w || !w->layer || w->layers <= 0 || w->width <= 0 || w->vocab <= 0 || !w->final_norm || !w->head) return COGS_E_INVALID;
    if (w->dtype != COGS_DT_BF16 && w->dtype != COGS_DT_F32) return COGS_E_INVALID;
    CogsDecoder* d = new (std::nothrow) CogsDecoder();
    if (!d) return COGS_E_HIP;
    auto fail = [&](cogs_status rc) { cogs_decoder_free(d); return rc; };
    d->w = *w;
    d->layers.assign(w->layer, w->layer + w->layers);
    d->w.layer = d->layers.data();
    d->wp = up(w->width, 64);
    d->vocabp = up(w->vocab, 4);
    std::vector<double> freq;
    std::vector<size_t> freq_at;
    const bool hyper = w->streams > 0;
    auto hyper_ok = [&](const cogs_hyper& c) { return !hyper || (c.in && c.out && c.mix); };
    for (int l = 0; l < w->layers; ++l) {
        const cogs_decoder_layer& L = d->layers[l];
        if (!L.norm1 || !hyper_ok(L.hyper1)) return fail(COGS_E_INVALID);
        Geom G{};
        int oin = 0, ocols = 0;
        if (L.mixer == COGS_MIX_LATENT) {
            const cogs_latent_mixer& m = L.latent;
            if (m.heads <= 0 || m.dim <= 0 || m.rot_dim < 2 || m.rot_dim % 2 || m.vdim <= 0 || m.q_rank <= 0 || m.kv_rank <= 0 ||
                !m.rot_freq || !m.in_w || !m.q_norm || !m.q_w || !m.kv_w || !m.k_abs || !m.o_w || m.kv_from >= l) return fail(COGS_E_INVALID);
            LatentGeom& g = G.lat;
            g.own = m.kv_from < 0;
            g.qrp = up(m.q_rank, 64); g.kvp = up(m.kv_rank, 64); g.rotc = up(m.rot_dim, 32); g.kvw = g.kvp + g.rotc;
            g.dn = up(m.dim, 8); g.dr = up(m.rot_dim, 8); g.dk = up(m.dim, 32); g.dq = g.dk + up(m.rot_dim, 32); g.dv = up(m.vdim, 16);
            g.oin = up(m.heads * g.dv, 64); g.headsp = up(m.heads, 4);
            g.ldt = g.qrp + (g.own ? g.kvw : 0) + (m.gated ? g.headsp : 0);
            g.kvcols = m.heads * (g.dn + g.dv);
            g.src = g.own ? l : m.kv_from;
            if (g.own) {
                if (!m.kv_norm) return fail(COGS_E_INVALID);
                G.rows_width = g.kvw;
            } else {
                const cogs_latent_mixer& s = d->layers[g.src].latent;
                if (d->layers[g.src].mixer != COGS_MIX_LATENT || !d->geom[g.src].lat.own || s.kv_rank != m.kv_rank || s.rot_dim != m.rot_dim)
                    return fail(COGS_E_INVALID);
            }
            // one table per distinct (head layout, rotation)
            const int n = m.rot_dim / 2;
            g.rope = -1;
            for (size_t s = 0; s < d->sets.size(); ++s) {
                const CogsRopeSet& R = d->sets[s];
                if (R.pairs == g.dq / 2 && R.first == g.dk / 2 && R.n == n && R.mag == m.rot_mag &&
                    memcmp(freq.data() + freq_at[s], m.rot_freq, n * sizeof(double)) == 0) g.rope = (int)s;
            }
            if (g.rope < 0) {
                g.rope = (int)d->sets.size();
                d->sets.push_back(CogsRopeSet{d->rope_width, g.dq / 2, g.dk / 2, n, m.rot_mag, nullptr});
                freq_at.push_back(freq.size());
                freq.insert(freq.end(), m.rot_freq, m.rot_freq + n);
                d->rope_width += g.dq;
                mx(d->max_pairs, g.dq / 2);
            }
            mx(d->max_t32, g.ldt); mx(d->max_cq, g.qrp); mx(d->max_q, m.heads * g.dq); mx(d->max_kvcols, g.kvcols);
            mx(d->max_kvw, g.kvw); mx(d->max_heads, m.heads);
            mx(d->max_qlat, (long)m.heads * g.kvw); mx(d->max_olat, (long)m.heads * g.kvp);
            oin = g.oin; ocols = m.heads * g.dv;
        } else if (L.mixer == COGS_MIX_ATTENTION) {
            const cogs_attn_mixer& m = L.attn;
            if (m.heads <= 0 || m.kv_heads <= 0 || m.heads % m.kv_heads || m.dim <= 0 || m.vdim <= 0 || !m.in_w || !m.o_w ||
                (m.dist_bias && m.dist_n <= 0)) return fail(COGS_E_INVALID);
            AttnGeom& g = G.att;
            g.dk = up(m.dim, 32); g.dv = up(m.vdim, 16); g.kvw = up(g.dk + g.dv, 32); g.oin = up(m.heads * g.dv, 64);
            g.ldt = (m.heads + m.kv_heads) * g.dk + m.kv_heads * g.dv;
            G.rows_width = m.kv_heads * g.kvw;
            mx(d->max_t32, g.ldt); mx(d->max_q, m.heads * g.dk);
            oin = g.oin; ocols = m.heads * g.dv;
        } else if (L.mixer == COGS_MIX_DELTA) {
            const cogs_delta_mixer& m = L.delta;
            if (m.heads <= 0 || m.kv_heads <= 0 || m.heads % m.kv_heads || m.dim <= 0 || m.vdim <= 0 || m.taps <= 0 || !m.in_w || !m.conv ||
                !m.neg_a || !m.dt_bias || !m.norm || !m.o_w) return fail(COGS_E_INVALID);
            DeltaGeom& g = G.del;
            g.dk = up(m.dim, 16); g.dv = up(m.vdim, 16); g.headsp = up(m.heads, 4); g.oin = up(m.heads * g.dv, 64);
            g.channels = 2 * m.kv_heads * g.dk + m.heads * g.dv;
            g.ldt = g.channels + m.heads * g.dv + 2 * g.headsp;
            G.state = (long)m.heads * g.dk * g.dv + (long)m.taps * g.channels;
            mx(d->max_t32, g.ldt); mx(d->max_dqk, m.kv_heads * g.dk); mx(d->max_dv, m.heads * g.dv); mx(d->max_dheads, m.heads);
            oin = g.oin; ocols = m.heads * g.dv;
        } else {
            return fail(COGS_E_INVALID);
        }
        mx(d->max_o, oin);
        if (ocols != oin) d->att_tail = true;
        if (L.mlp.ff > 0) {
            if (!L.norm2 || !L.mlp.up_w || !L.mlp.down_w || L.mlp.act < COGS_ACT_NONE || L.mlp.act > COGS_ACT_SWIGLU || !hyper_ok(L.hyper2))
                return fail(COGS_E_INVALID);
            mx(d->max_ff, up(L.mlp.ff, 64));
        }
        d->geom.push_back(G);
    }
    {   // the layer runs, each with rows and state of its own; borrowed rows are those of the source's latest run
        const bool loop = w->loop_times > 1;
        if (loop && (w->loop_start < 0 || w->loop_stop > w->layers || w->loop_start >= w->loop_stop)) return fail(COGS_E_INVALID);
        std::vector<long> at(w->layers, 0);
        auto run = [&](int l) {
            const Geom& G = d->geom[l];
            at[l] = d->cache_width;
            const bool borrows = d->layers[l].mixer == COGS_MIX_LATENT && !G.lat.own;
            d->runs.push_back(Run{l, borrows ? at[G.lat.src] : d->cache_width, d->state_floats});
            d->cache_width += G.rows_width;
            d->state_floats += G.state;
        };
        for (int l = 0; l < w->layers; ++l) {
            run(l);
            if (loop && l == w->loop_stop - 1)
                for (int t = 1; t < w->loop_times; ++t)
                    for (int m = w->loop_start; m < w->loop_stop; ++m) run(m);
        }
    }
    if (!d->sets.empty() && (hipMalloc(&d->freq_dev, freq.size() * sizeof(double)) != hipSuccess ||
                             hipMalloc(&d->sets_dev, d->sets.size() * sizeof(CogsRopeSet)) != hipSuccess)) return fail(COGS_E_HIP);
    for (size_t s = 0; s < d->sets.size(); ++s) d->sets[s].freq = d->freq_dev + freq_at[s];
    if (!d->sets.empty() && (
        hipMemcpy(d->freq_dev, freq.data(), freq.size() * sizeof(double), hipMemcpyHostToDevice) != hipSuccess ||
        hipMemcpy(d->sets_dev, d->sets.data(), d->sets.size() * sizeof(CogsRopeSet), hipMemcpyHostToDevice) != hipSuccess)) return fail(COGS_E_HIP);
    cogs_decoder_free(h->decoder);
    h->decoder = d;
    return COGS_OK;
}

cogs_status cogs_decoder_cache_width(cogs_handle h, int64_t* elements) {
    if (!h || !h->decoder || !elements) return COGS_E_INVALID;
    *elements = h->decoder->cache_width;
    return COGS_OK;
}

cogs_status cogs_decoder_state_bytes(cogs_handle h, int64_t* bytes) {
    if (!h || !h->decoder || !bytes) return COGS_E_INVALID;
    *bytes = h->decoder->state_floats * 4;
    return COGS_OK;
}

cogs_status cogs_decoder_workspace_bytes(cogs_handle h, int rows, int nseq, int64_t total_context, int n_want, size_t* bytes) {
    if (!h || !h->decoder || !bytes || rows <= 0 || nseq <= 0 || nseq > rows || total_context < rows || n_want < 0) return COGS_E_INVALID;
    if (total_context > 0x7fffffff) return COGS_E_INVALID;
    *bytes = carve(*h->decoder, rows, nseq, total_context, n_want, nullptr, 0).bytes;
    return COGS_OK;
}

cogs_status cogs_decoder_forward(cogs_handle h, cogs_stream stream, const void* embeds, cogs_kv* const* kv, const int32_t* lens, int nseq,
                                 const int32_t* want, int n_want, float* logits, float* streams, void* ws, size_t ws_bytes) {
    if (!h || !h->decoder || !embeds || !kv || !lens || nseq <= 0 || n_want < 0 || (n_want > 0 && (!want || !logits))) return COGS_E_INVALID;
    const CogsDecoder& d = *h->decoder;
    hipStream_t st = (hipStream_t)stream;
    std::vector<CogsSeq> seqs(nseq);
    int64_t rows = 0, C = 0;
    int max_new = 0, max_ctx = 0;
    for (int i = 0; i < nseq; ++i) {
        if (!kv[i] || (d.cache_width > 0 && !kv[i]->k) || (d.state_floats > 0 && !kv[i]->v) || lens[i] <= 0 || kv[i]->len < 0 || (int64_t)kv[i]->len + lens[i] > kv[i]->max_len) return COGS_E_INVALID;
        for (int j = 0; j < i; ++j)
            if (kv[j] == kv[i]) return COGS_E_INVALID;
        const int ctx = kv[i]->len + lens[i];
        if (d.w.max_positions > 0 && ctx > d.w.max_positions) return COGS_E_INVALID;
        seqs[i] = CogsSeq{(char*)kv[i]->k, (float*)kv[i]->v, kv[i]->max_len, (int)rows, lens[i], kv[i]->len, (int)C};
        rows += lens[i];
        C += ctx;
        max_new = lens[i] > max_new ? lens[i] : max_new;
        max_ctx = ctx > max_ctx ? ctx : max_ctx;
    }
    if (rows > 0x7fffffff || C > 0x7fffffff) return COGS_E_INVALID;
    for (int i = 0; i < n_want; ++i)
        if (want[i] < 0 || want[i] >= rows) return COGS_E_INVALID;
    const int S = (int)rows;
    Work k = carve(d, S, nseq, C, n_want, ws, ws_bytes);
    if (!ws || ws_bytes < k.bytes) return COGS_E_WORKSPACE;
    COGS_TRY(stage_h2d(h, st, k.seqs, seqs.data(), nseq * sizeof(CogsSeq)));
    if (n_want > 0) COGS_TRY(stage_h2d(h, st, k.want, want, (size_t)n_want * sizeof(int32_t)));
    Step s{h, st, d, k, seqs, S, nseq, max_new, max_ctx, C};
    {
        PROF(COGS_PROF_OTHER);
        COGS_TRY(cogs_k_seq_rows(st, k.seqs, nseq, S, k.rowseq, k.rowpos));
        if (!d.sets.empty()) COGS_TRY(cogs_k_rope_sets(st, k.rope, d.sets_dev, (int)d.sets.size(), d.max_pairs, k.rowpos, S));
        if (d.att_tail) COGS_TRY(cogs_k_zero(st, k.att, align_up((size_t)S * d.max_o * esize(d.w.dtype))));
    }
    COGS_TRY(s.stream(embeds, nullptr, nullptr, &d.layers[0].hyper1, d.layers[0].norm1, nullptr));
    for (size_t r = 0; r < d.runs.size(); ++r) {
        const cogs_decoder_layer& L = d.layers[d.runs[r].layer];
        const cogs_decoder_layer* next = r + 1 < d.runs.size() ? &d.layers[d.runs[r + 1].layer] : nullptr;
        float* sum = streams ? streams + r * S * d.wp : nullptr;
        COGS_TRY(s.mixer(d.runs[r]));
        const cogs_hyper* from = &L.hyper1;
        const float* gamma = L.norm1b;
        if (L.mlp.ff > 0) {
            COGS_TRY(s.stream(nullptr, L.norm1b, &L.hyper1, &L.hyper2, L.norm2, nullptr));
            COGS_TRY(s.mlp(d.runs[r].layer));
            from = &L.hyper2;
            gamma = L.norm2b;
        }
        COGS_TRY(s.stream(nullptr, gamma, from, next ? &next->hyper1 : nullptr, next ? next->norm1 : nullptr, sum));
    }
    for (int i = 0; i < nseq; ++i) kv[i]->len += lens[i];
    if (n_want > 0) {
        CogsStreamNorm a;
        a.x = k.x; a.streams = d.w.streams; a.out = k.hn; a.out_gamma = d.w.final_norm; a.pick = k.want; a.rows = n_want; a.H = d.w.width; a.Hp = d.wp; a.eps = d.w.eps;
        { PROF(COGS_PROF_NORM); COGS_TRY(cogs_k_stream_norm(st, d.w.dtype, a)); }
        CogsGemm g;
        g.A = k.hn; g.lda = d.wp; g.W = d.w.head; g.ldw = d.wp; g.C = logits; g.ldc = d.vocabp; g.M = n_want; g.N = d.vocabp; g.K = d.wp; g.out_f32 = 1;
        COGS_TRY(s.lin(g));
    }
    return COGS_OK;
}

}  // extern "C"
