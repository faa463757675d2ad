// Decoder over a list of layers that differ from each other: every entry names its mixer -- attention over a shared, a ranged or a
// latent cache, or a delta rule on a recurrent state -- with its own sizes, and a feed-forward or none.  The two sublayers run side by
// side on one norm, or one after the other on a norm each; a table may add something of the token's own to every layer:
//
//   side by side:         h = norm(x);  x += mult * (mixer(h) + Wdown . act(Wup h))
//   one after the other:  x += mult * mixer(norm(x));  x += mult * Wdown . act(Wup norm2(x))
//   side table:           y = Wproj (gelu(Wgate x) * table[token][layer]);  x += y / rms(y) * side_norm
//
// with the residual stream in fp32.  What reads h is one stacked matrix and what adds to x is one matrix (side by side: its columns
// are the mixer's outputs followed by the feed-forward's), so a layer is, per decode step, [norm + input projections + their
// activations], the mixer, [output projections + residual], then where they stand apart [norm + up + activation], [down + residual],
// and for the table [gate], [projection], whose norm and sum are part of the next launch that reads x.  A prompt takes the
// same products as GEMMs with the same epilogues, and the row-wise parts between them.
// Weights are bf16 or fp32; with fp32 weights every operand, the cached rows included, is fp32.
// The decode loop around a step is csrc/stepper.h; pages come from csrc/kv.h and states from csrc/rstate.h.
#include "dense.h"
#include "kv.h"
#include "rstate.h"
#include "stepper.h"

#include <algorithm>
#include <cmath>

namespace {

constexpr int kSliceTokens = 8192;  // prompts are run in slices of at most this many tokens (a bound for the buffers)
constexpr int kWantRows = 256;      // rows of logits per head product
constexpr int kStepCols = 5;        // fp32 projections of a decode step at most

struct Layer {
    skn_hybrid_layer p;
    skn_dense_mat in, out, decay, gate, up, down, side_gate, side_proj;
    int hd = 0, off_ff = 0;  // mixer output columns, first feed-forward column of `out` (side by side)
    skn_shared_attn shared;
    skn_ranged_attn ranged;
    skn_latent_attn latent;
    skn_channel_delta channel;
    double* rot_freq = nullptr;
    skn_kv* kv = nullptr;  // null in the delta rules
    bool owns_kv = false;  // (a layer may read another one's cache)
    skn_rstate* state = nullptr;
};

}  // namespace

struct skn_hybrid {
    skn_hybrid_config cfg;
    std::vector<Layer> layers;
    skn_dense_mat head;
    const void* embed = nullptr;
    const float* final_norm = nullptr;
    const void* side = nullptr;
    skn_stepper step;
    int pos = 0;
    int width_pad = 0, max_cols = 0, max_out = 0, max_ff = 0, max_rank = 0, max_attn = 0, max_lat = 0, max_heads = 0, prompt_cols = 0, side_pad = 0;
    double* inv_freq = nullptr;
    // decode-step buffers (two for x: a launch that adds a layer's side term writes the other one)
    float *x = nullptr, *x2 = nullptr, *cols = nullptr, *mix = nullptr, *mid = nullptr, *rank = nullptr, *rank2 = nullptr, *logits = nullptr, *opart = nullptr,
          *ml = nullptr, *qprep = nullptr, *sg = nullptr, *sy = nullptr;
    // prompt buffers (grown to the longest slice seen)
    int cap = 0;
    float *px = nullptr, *pcols = nullptr, *pq = nullptr, *plat = nullptr, *ppack = nullptr, *py = nullptr, *plogits = nullptr;
    void *ph = nullptr, *pa = nullptr, *prank = nullptr, *prank2 = nullptr, *psg = nullptr, *pwant_h = nullptr;
    int32_t *ptok = nullptr, *pwant = nullptr;
    skn_latent_ws latent_ws;
    std::vector<void*> owned;
};

namespace {

template <typename T>
int dev_alloc(skn_ctx* ctx, skn_hybrid* m, T** p, size_t bytes) {
    bytes = bytes < 256 ? 256 : bytes;
    hipError_t e = hipMalloc((void**)p, bytes);
    if (e != hipSuccess) {
        (void)hipGetLastError();
        return skn_fail(ctx, SKN_ERR_OOM, "skn_hybrid: %zu bytes: %s", bytes, hipGetErrorString(e));
    }
    m->owned.push_back((void*)*p);
    // (padding columns are multiplied by zero weights: they only have to be finite)
    SKN_HIP(ctx, hipMemsetAsync((void*)*p, 0, bytes, ctx->stream));
    return SKN_OK;
}

template <typename T>
void dev_release(skn_hybrid* m, T** p) {
    if (!*p) return;
    m->owned.erase(std::remove(m->owned.begin(), m->owned.end(), (void*)*p), m->owned.end());
    (void)hipFree((void*)*p);
    *p = nullptr;
}

size_t elem_bytes(const skn_hybrid* m) { return m->cfg.weight_type == SKN_TYPE_F32 ? 4 : 2; }

int ensure_prompt_buffers(skn_ctx* ctx, skn_hybrid* m, int T) {
    if (T <= m->cap) return SKN_OK;
    SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    m->cap = 0;
    dev_release(m, &m->px); dev_release(m, &m->pcols); dev_release(m, &m->pq); dev_release(m, &m->ppack); dev_release(m, &m->plat); dev_release(m, &m->py);
    dev_release(m, &m->ph); dev_release(m, &m->pa); dev_release(m, &m->prank); dev_release(m, &m->prank2); dev_release(m, &m->psg); dev_release(m, &m->ptok);
    const size_t es = elem_bytes(m), t = T;
    size_t pack = 0;
    for (const Layer& L : m->layers)
        if (L.state) pack = std::max(pack, L.p.mixer == SKN_MIX_CHANNEL_DELTA ? skn_gated_delta_pack_floats(L.state, T) : skn_delta_pack_floats(L.state, T));
    SKN_TRY(dev_alloc(ctx, m, &m->px, t * m->width_pad * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->pcols, m->prompt_cols * t * m->max_cols * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->pq, t * m->max_attn * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->plat, t * m->max_lat * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->ppack, pack * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->ph, t * m->width_pad * es));
    SKN_TRY(dev_alloc(ctx, m, &m->pa, t * m->max_out * es));
    SKN_TRY(dev_alloc(ctx, m, &m->prank, t * m->max_rank * es));
    SKN_TRY(dev_alloc(ctx, m, &m->prank2, t * m->max_rank * es));
    SKN_TRY(dev_alloc(ctx, m, &m->psg, t * m->side_pad * es));
    SKN_TRY(dev_alloc(ctx, m, &m->py, m->side ? t * m->width_pad * 4 : 0));
    SKN_TRY(dev_alloc(ctx, m, &m->ptok, t * sizeof(int32_t)));
    m->cap = T;
    return SKN_OK;
}

void add_seg(skn_dense_out& o, int row0, int rows, int op, void* out, int ldo, int type, float p0 = 0.f, float p1 = 0.f) {
    o.seg[o.nseg++] = {row0, rows, op, p0, p1, out, ldo, type};
}

int act_op(const Layer& L) { return L.p.act == SKN_ACT_GELU ? SKN_OP_GELU : SKN_OP_XIELU; }

// Where the rows of a layer's input matrix go, in the order of the header.  cols: the fp32 ones (segment i at cols + i *
// col_stride, rows of ldc); the low-rank ones to rank and rank2, the feed-forward's to mid, all of mid_type.
struct InputDest {
    float* cols;
    int64_t col_stride;
    int ldc;
    void *rank, *rank2;
    int ldr, ldr2;
    void* mid;
    int ldm, mid_type;
};
skn_dense_out input_segments(const Layer& L, const InputDest& d) {
    const skn_hybrid_layer& p = L.p;
    skn_dense_out o;
    int row = 0;
    auto put = [&](int rows, int op, void* out, int ld, int type, float p0 = 0.f, float p1 = 0.f) {
        add_seg(o, row, rows, op, out, ld, type, p0, p1);
        row += skn_pad_rows(rows);
    };
    auto col = [&](int i, int rows, int op = SKN_OP_NONE) { put(rows, op, d.cols + i * d.col_stride, d.ldc, SKN_TYPE_F32); };
    switch (p.mixer) {
        case SKN_MIX_SHARED_ATTN:
            col(0, L.hd);
            col(1, p.kv_heads * p.dim);
            break;
        case SKN_MIX_RANGED_ATTN:
            col(0, p.heads * p.dim);
            col(1, p.kv_heads * p.dim);
            col(2, p.kv_heads * p.vdim);
            col(3, L.hd, SKN_OP_SIGMOID);
            break;
        case SKN_MIX_LATENT_ATTN:
            col(0, p.heads * (p.dim + p.rot_dims));
            if (L.owns_kv) col(1, p.kv_rank + p.rot_dims);
            break;
        case SKN_MIX_CHANNEL_DELTA:
            col(0, p.kv_heads * p.dim);
            col(1, p.kv_heads * p.dim);
            col(2, L.hd);
            col(3, p.heads, SKN_OP_SIGMOID);
            put(p.rank, SKN_OP_NONE, d.rank, d.ldr, d.mid_type);
            put(p.rank_gate, SKN_OP_NONE, d.rank2, d.ldr2, d.mid_type);
            break;
        default:
            for (int i = 0; i < 5; i++) col(i, L.hd, i < 3 ? SKN_OP_NONE : SKN_OP_SIGMOID);
            put(p.rank, SKN_OP_TANH, d.rank, d.ldr, d.mid_type);
    }
    if (p.ff && !p.norm2) put(p.ff, act_op(L), d.mid, d.ldm, d.mid_type, p.act_pos, p.act_neg);
    return o;
}

skn_dense_out residual(const skn_hybrid* m, float* x) {
    skn_dense_out o;
    o.resid = x;
    o.ldr = m->width_pad;
    o.resid_rows = m->cfg.width;
    o.mult = m->cfg.residual_mult;
    return o;
}

// the side table's gate: rows of `out`, times the tokens' parts for layer l
skn_dense_out side_segment(const skn_hybrid* m, int l, const int32_t* tokens, void* out, int ldo, int type) {
    skn_dense_out o;
    add_seg(o, 0, m->cfg.side_dim, SKN_OP_GELU, out, ldo, type);
    o.mul_seg = 0;
    o.mul_table = m->side;
    o.mul_type = m->cfg.weight_type;
    o.mul_ld = skn_pad_cols(m->cfg.n_layer * m->cfg.side_dim);
    o.mul_col = l * m->cfg.side_dim;
    o.mul_tokens = tokens;
    return o;
}

// ---- decode -----------------------------------------------------------------------------------------------------------

// the mixer of a decode step, from m->cols to m->mix, or to the split partials that `src` then names
int mixer_step(skn_ctx* ctx, skn_hybrid* m, Layer& L, int max_ctx, skn_matvec_src& src) {
    const float* col[kStepCols];
    for (int i = 0; i < kStepCols; i++) col[i] = m->cols + (int64_t)i * m->max_cols;
    const int32_t* state = m->step.state;
    auto merge = [&](int splits, int heads, int dim) {
        if (splits <= 1) return;
        src.mode = SKN_XSRC_MERGE;
        src.x0 = m->opart;
        src.ml = m->ml;
        src.splits = splits;
        src.heads = heads;
        src.dim = dim;
        src.dim_pad = L.kv->head_dim;
    };
    switch (L.p.mixer) {
        case SKN_MIX_SHARED_ATTN: {
            const int splits = skn_shared_attn_splits(ctx, L.kv, L.shared.n_head, max_ctx);
            SKN_TRY(skn_shared_attn_step(ctx, L.kv, 0, L.shared, col[0], col[1], state, splits, m->opart, m->ml, m->mix));
            merge(splits, L.shared.n_head, L.kv->dim);
            return SKN_OK;
        }
        case SKN_MIX_RANGED_ATTN: {
            skn_range r;
            r.kind = L.ranged.mask;
            r.size = L.ranged.mask_size;
            const int splits = skn_ranged_splits(ctx, L.p.heads, 16 * 512 / L.kv->head_dim * 4, r, max_ctx);
            SKN_TRY(skn_ranged_attn_step(ctx, L.kv, 0, L.ranged, col[0], col[1], col[2], col[3], state, splits, m->opart, m->ml, m->mix));
            merge(splits, L.p.heads, L.p.vdim);
            if (splits > 1) {
                src.sink = L.ranged.sink;
                src.gate = col[3];
            }
            return SKN_OK;
        }
        case SKN_MIX_LATENT_ATTN:
            return skn_latent_step(ctx, L.kv, 0, L.latent, col[0], L.owns_kv ? col[1] : nullptr, state, skn_latent_splits(ctx, L.kv, L.latent, max_ctx), m->qprep,
                                   m->opart, m->ml, m->mix);
        case SKN_MIX_CHANNEL_DELTA: {
            skn_gated_step d;
            d.q = col[0], d.k = col[1], d.v = col[2], d.beta = col[3];
            d.a_low = m->rank, d.g_low = m->rank2;
            d.w_a = L.decay.w, d.w_g = L.gate.w;
            d.w_type = L.decay.type;
            d.rank_a_pad = L.decay.k_pad, d.rank_g_pad = L.gate.k_pad;
            d.bias_a = L.decay.bias;
            d.norm = L.p.o_norm;
            d.eps = m->cfg.norm_eps;
            d.state = state;
            d.y = m->mix;
            return skn_gated_step_launch(ctx, L.state, 0, L.channel, d);
        }
        default: {
            skn_delta_step d;
            d.r = col[0], d.k = col[1], d.v = col[2], d.g = col[3], d.a = col[4];
            d.t = m->rank;
            d.w2 = L.decay.w;
            d.w2_type = L.decay.type;
            d.rank = L.p.rank;
            d.rank_pad = L.decay.k_pad;
            d.b2 = L.decay.bias;
            d.norm = L.p.o_norm;
            d.eps = m->cfg.norm_eps;
            d.y = m->mix;
            return skn_delta_step_launch(ctx, L.state, 0, d);
        }
    }
}

int decode_step(skn_ctx* ctx, skn_hybrid* m, int max_ctx) {
    const skn_hybrid_config& c = m->cfg;
    SKN_TRY(skn_embed_rows(ctx, m->embed, c.weight_type, m->width_pad, m->step.state, m->step.state + 1, c.sinusoid ? m->inv_freq : nullptr, c.embed_scale, 1,
                           c.width, m->x, m->width_pad));
    float *x = m->x, *other = m->x2;
    const Layer* pending = nullptr;  // the layer whose side term (its projection in m->sy) x still lacks
    skn_matvec_src norm;
    norm.k0 = c.width;
    norm.groups = c.norm_groups;
    norm.eps = c.norm_eps;
    auto normed = [&](const float* w) {
        norm.mode = pending ? SKN_XSRC_ADD_NORM : SKN_XSRC_GROUP_NORM;
        norm.x0 = x;
        norm.norm_w = w;
        if (pending) {
            norm.add = m->sy;
            norm.add_w = pending->p.side_norm;
            norm.x_out = other;
            std::swap(x, other);
            pending = nullptr;
        }
    };
    for (int l = 0; l < c.n_layer; l++) {
        Layer& L = m->layers[l];
        skn_dense_out in = input_segments(L, {m->cols, m->max_cols, m->max_cols, m->rank, m->rank2, m->max_rank, m->max_rank, m->mid, m->max_ff, SKN_TYPE_F32});
        if (L.p.mixer == SKN_MIX_SHARED_ATTN) {
            in.cache_seg = 1;
            in.k_pool = L.kv->k_pool;
            in.elem_type = L.kv->elem_type;
            in.kv_heads = L.kv->n_head;
            in.dim = L.kv->dim;
            in.dim_pad = L.kv->head_dim;
            in.page_tokens = L.kv->page_tokens;
            in.page_table = L.kv->page_table_dev;
            in.pos_dev = m->step.state + 1;
        }
        normed(L.p.norm);
        SKN_TRY(skn_dense_matvec(ctx, L.in, norm, in));
        skn_matvec_src src;
        src.x0 = m->mix;
        src.k0 = L.hd;
        if (L.p.ff && !L.p.norm2) {
            src.x1 = m->mid;
            src.off1 = L.off_ff;
            src.k1 = L.p.ff;
        }
        SKN_TRY(mixer_step(ctx, m, L, max_ctx, src));
        SKN_TRY(skn_dense_matvec(ctx, L.out, src, residual(m, x)));
        if (L.p.ff && L.p.norm2) {
            normed(L.p.norm2);
            skn_dense_out up;
            add_seg(up, 0, L.p.ff, act_op(L), m->mid, m->max_ff, SKN_TYPE_F32, L.p.act_pos, L.p.act_neg);
            SKN_TRY(skn_dense_matvec(ctx, L.up, norm, up));
            skn_matvec_src mid;
            mid.x0 = m->mid;
            mid.k0 = L.p.ff;
            SKN_TRY(skn_dense_matvec(ctx, L.down, mid, residual(m, x)));
        }
        if (m->side) {
            skn_matvec_src plain;
            plain.x0 = x;
            plain.k0 = c.width;
            SKN_TRY(skn_dense_matvec(ctx, L.side_gate, plain, side_segment(m, l, m->step.state, m->sg, m->side_pad, SKN_TYPE_F32)));
            plain.x0 = m->sg;
            plain.k0 = c.side_dim;
            skn_dense_out y;
            add_seg(y, 0, c.width, SKN_OP_NONE, m->sy, m->width_pad, SKN_TYPE_F32);
            SKN_TRY(skn_dense_matvec(ctx, L.side_proj, plain, y));
            pending = &L;
        }
    }
    normed(m->final_norm);
    skn_dense_out lg;
    add_seg(lg, 0, c.vocab, SKN_OP_NONE, m->logits, skn_pad_cols(c.vocab), SKN_TYPE_F32);
    SKN_TRY(skn_dense_matvec(ctx, m->head, norm, lg));
    return skn_stepper_pick(ctx, &m->step, m->logits, c.vocab, 1);
}

int run_steps(skn_ctx* ctx, skn_hybrid* m, int first_token, int n_steps, int32_t* tokens_out_host) {
    for (Layer& L : m->layers)
        if (L.owns_kv) SKN_TRY(skn_kv_reserve(ctx, L.kv, 0, m->pos + n_steps));
    // the step is captured for contexts up to a power of two (the attention's split counts), again when a run passes it
    int max_ctx = 128;
    while (max_ctx < m->pos + n_steps) max_ctx *= 2;
    SKN_TRY(skn_stepper_run(ctx, &m->step, first_token, m->pos, n_steps, max_ctx, [&]() { return decode_step(ctx, m, max_ctx); }, tokens_out_host));
    m->pos += n_steps;
    for (Layer& L : m->layers)
        if (L.owns_kv) L.kv->len[0] = m->pos;
    return SKN_OK;
}

// ---- prompts ----------------------------------------------------------------------------------------------------------

// the mixer over the slice's rows, from m->pcols to the first columns of m->pa
int mixer_rows(skn_ctx* ctx, skn_hybrid* m, Layer& L, int n, int pos0, int64_t stride) {
    const skn_hybrid_config& c = m->cfg;
    const int type = c.weight_type, ld = m->max_cols, lda = L.out.k_pad;
    auto col = [&](int i) { return m->pcols + i * stride; };
    switch (L.p.mixer) {
        case SKN_MIX_SHARED_ATTN:
            SKN_TRY(skn_shared_prep_rows(ctx, L.kv, 0, L.shared, col(0), ld, col(1), ld, n, pos0, m->pq));
            return skn_shared_attn_rows(ctx, L.kv, 0, L.shared, m->pq, n, pos0, m->pa, lda, type);
        case SKN_MIX_RANGED_ATTN:
            SKN_TRY(skn_ranged_prep_rows(ctx, L.kv, 0, L.ranged, col(0), ld, col(1), ld, col(2), ld, n, pos0, m->pq));
            return skn_ranged_attn_rows(ctx, L.kv, 0, L.ranged, m->pq, n, pos0, col(3), ld, m->pa, lda, type);
        case SKN_MIX_LATENT_ATTN:
            return skn_latent_rows(ctx, L.kv, 0, L.latent, col(0), ld, L.owns_kv ? col(1) : nullptr, ld, n, pos0, m->pq, m->plat, &m->latent_ws, m->pa, lda, type);
        case SKN_MIX_CHANNEL_DELTA: {
            skn_dense_out z, g;
            add_seg(z, 0, L.p.heads * L.p.dim, SKN_OP_NONE, col(4), ld, SKN_TYPE_F32);
            SKN_TRY(skn_dense_gemm(ctx, L.decay, m->prank, L.decay.k_pad, n, z));
            add_seg(g, 0, L.hd, SKN_OP_SIGMOID, col(5), ld, SKN_TYPE_F32);
            SKN_TRY(skn_dense_gemm(ctx, L.gate, m->prank2, L.gate.k_pad, n, g));
            SKN_TRY(skn_gated_delta_rows(ctx, L.state, 0, L.channel, col(0), col(1), col(2), col(3), col(4), ld, n, pos0, col(6), col(7), col(8), m->ppack, col(9)));
            return skn_delta_gate_rows(ctx, col(9), col(5), ld, L.p.o_norm, n, L.p.heads, L.p.vdim, c.norm_eps, m->pa, lda, type);
        }
        default: {
            skn_dense_out w;
            add_seg(w, 0, L.hd, SKN_OP_DECAY, col(5), ld, SKN_TYPE_F32);
            SKN_TRY(skn_dense_gemm(ctx, L.decay, m->prank, L.decay.k_pad, n, w));
            float* o = col(5);  // (the decays are packed before the scan writes its outputs over them)
            SKN_TRY(skn_delta_rows(ctx, L.state, 0, col(0), col(1), col(2), col(5), col(4), ld, n, m->ppack, o));
            return skn_delta_gate_rows(ctx, o, col(3), ld, L.p.o_norm, n, L.p.heads, L.p.dim, c.norm_eps, m->pa, lda, type);
        }
    }
}

// n tokens (device ids in m->ptok) through all layers; the residual rows are left in m->px
int run_slice(skn_ctx* ctx, skn_hybrid* m, int n) {
    const skn_hybrid_config& c = m->cfg;
    const int pos0 = m->pos, type = c.weight_type;
    for (Layer& L : m->layers)
        if (L.owns_kv) SKN_TRY(skn_kv_reserve(ctx, L.kv, 0, pos0 + n));
    SKN_TRY(skn_stepper_set(ctx, &m->step, 0, pos0));
    SKN_TRY(skn_embed_rows(ctx, m->embed, type, m->width_pad, m->ptok, m->step.state + 1, c.sinusoid ? m->inv_freq : nullptr, c.embed_scale, n, c.width, m->px,
                           m->width_pad));
    const int64_t stride = (int64_t)n * m->max_cols;
    const Layer* pending = nullptr;  // as in decode_step; its projections are in m->py
    for (int l = 0; l < c.n_layer; l++) {
        Layer& L = m->layers[l];
        if (pending)
            SKN_TRY(skn_add_norm_rows(ctx, m->px, m->width_pad, m->py, m->width_pad, pending->p.side_norm, L.p.norm, n, c.width, c.norm_eps, m->ph, m->width_pad, type));
        else SKN_TRY(skn_group_norm_rows(ctx, m->px, m->width_pad, nullptr, L.p.norm, n, c.width, c.norm_groups, c.norm_eps, m->ph, m->width_pad, type));
        void* mid = (uint8_t*)m->pa + (size_t)L.off_ff * elem_bytes(m);  // (the output product's activations: mixer columns, then the feed-forward's)
        const skn_dense_out in = input_segments(L, {m->pcols, stride, m->max_cols, m->prank, m->prank2, L.decay.k_pad, L.gate.k_pad, mid, L.out.k_pad, type});
        SKN_TRY(skn_dense_gemm(ctx, L.in, m->ph, m->width_pad, n, in));
        SKN_TRY(mixer_rows(ctx, m, L, n, pos0, stride));
        if (L.owns_kv) L.kv->len[0] = pos0 + n;
        SKN_TRY(skn_dense_gemm(ctx, L.out, m->pa, L.out.k_pad, n, residual(m, m->px)));
        if (L.p.ff && L.p.norm2) {
            SKN_TRY(skn_group_norm_rows(ctx, m->px, m->width_pad, nullptr, L.p.norm2, n, c.width, c.norm_groups, c.norm_eps, m->ph, m->width_pad, type));
            skn_dense_out up;
            add_seg(up, 0, L.p.ff, act_op(L), m->pa, L.down.k_pad, type, L.p.act_pos, L.p.act_neg);
            SKN_TRY(skn_dense_gemm(ctx, L.up, m->ph, m->width_pad, n, up));
            SKN_TRY(skn_dense_gemm(ctx, L.down, m->pa, L.down.k_pad, n, residual(m, m->px)));
        }
        if (m->side) {
            const void* x = m->px;
            if (type == SKN_TYPE_BF16) {
                SKN_TRY(skn_bf16_rows(ctx, m->px, m->width_pad, n, m->ph));
                x = m->ph;
            }
            SKN_TRY(skn_dense_gemm(ctx, L.side_gate, x, m->width_pad, n, side_segment(m, l, m->ptok, m->psg, m->side_pad, type)));
            skn_dense_out y;
            add_seg(y, 0, c.width, SKN_OP_NONE, m->py, m->width_pad, SKN_TYPE_F32);
            SKN_TRY(skn_dense_gemm(ctx, L.side_proj, m->psg, m->side_pad, n, y));
            pending = &L;
        }
    }
    if (pending)
        SKN_TRY(skn_add_norm_rows(ctx, m->px, m->width_pad, m->py, m->width_pad, pending->p.side_norm, nullptr, n, c.width, c.norm_eps, nullptr, 0, type));
    m->pos = pos0 + n;
    return SKN_OK;
}

// logits of rows want[0..n) of the slice in m->px -> host [n][vocab]
int slice_logits(skn_ctx* ctx, skn_hybrid* m, const int32_t* want, int n, float* host) {
    const skn_hybrid_config& c = m->cfg;
    const int ldv = skn_pad_cols(c.vocab);
    if (!m->plogits) {
        SKN_TRY(dev_alloc(ctx, m, &m->pwant, kWantRows * sizeof(int32_t)));
        SKN_TRY(dev_alloc(ctx, m, &m->pwant_h, (size_t)kWantRows * m->width_pad * elem_bytes(m)));
        SKN_TRY(dev_alloc(ctx, m, &m->plogits, (size_t)kWantRows * ldv * sizeof(float)));
    }
    for (int i = 0; i < n; i += kWantRows) {
        const int k = std::min(kWantRows, n - i);
        SKN_HIP(ctx, hipMemcpyAsync(m->pwant, want + i, (size_t)k * sizeof(int32_t), hipMemcpyHostToDevice, ctx->stream));
        SKN_TRY(skn_group_norm_rows(ctx, m->px, m->width_pad, m->pwant, m->final_norm, k, c.width, c.norm_groups, c.norm_eps, m->pwant_h, m->width_pad,
                                    c.weight_type));
        skn_dense_out lg;
        add_seg(lg, 0, c.vocab, SKN_OP_NONE, m->plogits, ldv, SKN_TYPE_F32);
        SKN_TRY(skn_dense_gemm(ctx, m->head, m->pwant_h, m->width_pad, k, lg));
        SKN_HIP(ctx, hipMemcpy2DAsync(host + (size_t)i * c.vocab, (size_t)c.vocab * 4, m->plogits, (size_t)ldv * 4, (size_t)c.vocab * 4, k,
                                      hipMemcpyDeviceToHost, ctx->stream));
        SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    }
    return SKN_OK;
}

// a prompt or a portion of one, in slices; logits of the wanted tokens (ascending) to the host.  *last: rows of the last
// slice, whose residual rows are still in m->px.
int run_prompt(skn_ctx* ctx, skn_hybrid* m, const int32_t* tokens, int n, const int32_t* want, int n_want, float* logits_host, int* last) {
    int w = 0;
    std::vector<int32_t> rows;
    for (int t0 = 0; t0 < n; t0 += kSliceTokens) {
        const int k = std::min(kSliceTokens, n - t0);
        SKN_TRY(ensure_prompt_buffers(ctx, m, k));
        SKN_HIP(ctx, hipMemcpyAsync(m->ptok, tokens + t0, (size_t)k * sizeof(int32_t), hipMemcpyHostToDevice, ctx->stream));
        SKN_TRY(run_slice(ctx, m, k));
        rows.clear();
        const int w0 = w;
        while (w < n_want && want[w] < t0 + k) rows.push_back(want[w++] - t0);
        if (!rows.empty()) SKN_TRY(slice_logits(ctx, m, rows.data(), (int)rows.size(), logits_host + (size_t)w0 * m->cfg.vocab));
        *last = k;
    }
    return SKN_OK;
}

int check_tokens(skn_ctx* ctx, const skn_hybrid* m, const int32_t* tokens, int n) {
    SKN_REQUIRE(ctx, m->pos + n <= m->cfg.max_tokens, SKN_ERR_POOL, "sequence is full (%d tokens, capacity %d)", m->pos + n, m->cfg.max_tokens);
    for (int i = 0; i < n; i++)
        SKN_REQUIRE(ctx, tokens[i] >= 0 && tokens[i] < m->cfg.vocab, SKN_ERR_RANGE, "skn_hybrid: token %d of a vocabulary of %d", tokens[i], m->cfg.vocab);
    return SKN_OK;
}

// layer l of `layers`
int check_layer(skn_ctx* ctx, const skn_hybrid_config& c, const skn_hybrid_layer* layers, int l) {
    const skn_hybrid_layer& p = layers[l];
    SKN_REQUIRE(ctx, p.mixer >= SKN_MIX_SHARED_ATTN && p.mixer <= SKN_MIX_CHANNEL_DELTA, SKN_ERR_TYPE, "skn_hybrid_create: layer %d has an unknown mixer (%d)", l, p.mixer);
    SKN_REQUIRE(ctx, p.heads > 0 && p.dim > 0 && p.dim <= 256 && p.ff >= 0, SKN_ERR_SHAPE, "skn_hybrid_create: layer %d: %d heads of %d (at most 256)", l,
                p.heads, p.dim);
    SKN_REQUIRE(ctx, p.norm && p.w_in && p.b_in && p.w_out && p.b_out, SKN_ERR_ARG, "skn_hybrid_create: layer %d has a null weight", l);
    const uintptr_t all = (uintptr_t)p.w_in | (uintptr_t)p.w_out | (uintptr_t)p.norm | (uintptr_t)p.b_in | (uintptr_t)p.b_out | (uintptr_t)p.w_decay |
                          (uintptr_t)p.norm2 | (uintptr_t)p.w_up | (uintptr_t)p.w_down | (uintptr_t)p.w_latent | (uintptr_t)p.w_gate | (uintptr_t)p.side_gate |
                          (uintptr_t)p.side_proj | (uintptr_t)p.side_norm;
    SKN_REQUIRE(ctx, (all & 15) == 0, SKN_ERR_ARG, "skn_hybrid_create: the weights of layer %d must be 16-byte aligned", l);
    SKN_REQUIRE(ctx, !p.norm2 || p.ff == 0 || (p.w_up && p.w_down), SKN_ERR_ARG, "skn_hybrid_create: layer %d has no feed-forward weights", l);
    SKN_REQUIRE(ctx, p.act == SKN_ACT_XIELU || p.act == SKN_ACT_GELU, SKN_ERR_TYPE, "skn_hybrid_create: layer %d has an unknown activation (%d)", l, p.act);
    SKN_REQUIRE(ctx, c.side_dim == 0 || (p.side_gate && p.side_proj && p.side_norm), SKN_ERR_ARG, "skn_hybrid_create: layer %d has no weights for the side table", l);
    const bool mask_ok = p.mask == SKN_MASK_CAUSAL || ((p.mask == SKN_MASK_WINDOW || p.mask == SKN_MASK_CHUNK) && p.mask_size > 0);
    const bool rot_ok = p.rot_dims >= 0 && p.rot_dims % 2 == 0 && (p.rot_dims == 0 || p.rot_base > 0.0);
    if (p.mixer == SKN_MIX_SHARED_ATTN || p.mixer == SKN_MIX_RANGED_ATTN || p.mixer == SKN_MIX_CHANNEL_DELTA)
        SKN_REQUIRE(ctx, p.kv_heads > 0 && p.heads % p.kv_heads == 0, SKN_ERR_SHAPE, "skn_hybrid_create: layer %d: kv_heads (%d) must divide heads (%d)", l,
                    p.kv_heads, p.heads);
    if (p.mixer >= SKN_MIX_RANGED_ATTN)
        SKN_REQUIRE(ctx, p.vdim > 0 && p.vdim <= 256, SKN_ERR_SHAPE, "skn_hybrid_create: layer %d: values of %d elements (at most 256)", l, p.vdim);
    switch (p.mixer) {
        case SKN_MIX_SHARED_ATTN:
            SKN_REQUIRE(ctx, p.q_norm && p.k_norm && (p.temp_coef == 0.f || p.temp_every > 0.f), SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad attention parameters", l);
            break;
        case SKN_MIX_RANGED_ATTN:
            SKN_REQUIRE(ctx, mask_ok && rot_ok && p.rot_dims <= p.dim, SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad attention parameters", l);
            break;
        case SKN_MIX_LATENT_ATTN: {
            SKN_REQUIRE(ctx, mask_ok && rot_ok && p.w_latent && p.kv_rank > 0, SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad latent attention parameters", l);
            const int j = p.kv_from;
            SKN_REQUIRE(ctx, j < l && (j >= 0 || p.latent_norm), SKN_ERR_ARG, "skn_hybrid_create: layer %d reads the cache of layer %d", l, j);
            SKN_REQUIRE(ctx, j < 0 || (layers[j].mixer == SKN_MIX_LATENT_ATTN && layers[j].kv_from < 0 && layers[j].kv_rank == p.kv_rank &&
                                       layers[j].rot_dims == p.rot_dims && layers[j].rot_base == p.rot_base),
                        SKN_ERR_SHAPE, "skn_hybrid_create: layer %d cannot read the cache of layer %d", l, j);
            break;
        }
        case SKN_MIX_CHANNEL_DELTA:
            SKN_REQUIRE(ctx, p.rank > 0 && p.rank_gate > 0 && p.w_decay && p.b_decay && p.w_gate && p.o_norm && p.conv && p.decay_rate && p.taps > 0, SKN_ERR_ARG,
                        "skn_hybrid_create: layer %d: bad delta rule parameters", l);
            break;
        default:
            SKN_REQUIRE(ctx, p.rank > 0 && p.w_decay && p.b_decay && p.o_norm, SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad delta rule parameters", l);
    }
    return SKN_OK;
}

int build_layer(skn_ctx* ctx, skn_hybrid* m, int l) {
    const skn_hybrid_config& c = m->cfg;
    Layer& L = m->layers[l];
    const skn_hybrid_layer& p = L.p;
    const int cache_type = c.weight_type == SKN_TYPE_F32 ? SKN_TYPE_F32 : SKN_TYPE_F16, type = c.weight_type;
    auto mat = [&](const void* w, int rows, int cols, const float* bias = nullptr) { return skn_dense_mat{w, type, skn_pad_rows(rows), skn_pad_cols(cols), bias}; };
    int rows = 0;
    auto in_rows = [&](int n) {
        rows += skn_pad_rows(n);
        m->max_cols = std::max(m->max_cols, skn_pad_cols(n));
    };
    L.hd = p.heads * (p.mixer >= SKN_MIX_RANGED_ATTN ? p.vdim : p.dim);
    in_rows(L.hd);  // (values, gate or query)
    if ((p.mixer == SKN_MIX_RANGED_ATTN || p.mixer == SKN_MIX_LATENT_ATTN) && p.rot_dims > 0) {
        std::vector<double> f(p.rot_dims / 2);
        for (int i = 0; i < p.rot_dims / 2; i++) f[i] = pow(p.rot_base, -2.0 * i / p.rot_dims);
        SKN_TRY(dev_alloc(ctx, m, &L.rot_freq, f.size() * sizeof(double)));
        SKN_TRY(skn_upload(ctx, L.rot_freq, f.data(), f.size() * sizeof(double)));
    }
    int prompt_cols = 4;
    switch (p.mixer) {
        case SKN_MIX_SHARED_ATTN:
            in_rows(p.kv_heads * p.dim);
            L.shared = {p.heads, p.scale, p.temp_coef, p.temp_every, c.norm_eps, p.q_norm, p.k_norm};
            SKN_TRY(skn_kv_create_shared(ctx, 1, p.kv_heads, p.dim, cache_type, c.page_tokens, c.max_tokens, &L.kv));
            break;
        case SKN_MIX_RANGED_ATTN:
            in_rows(p.heads * p.dim);
            in_rows(p.kv_heads * p.dim);
            in_rows(p.kv_heads * p.vdim);
            L.ranged = {p.heads, p.mask, p.mask_size, p.sink, p.rot_dims, p.scale, p.softcap, c.norm_eps, p.q_norm, p.k_norm, L.rot_freq};
            SKN_TRY(skn_kv_create_ranged(ctx, 1, p.kv_heads, p.dim, p.vdim, cache_type, c.page_tokens, c.max_tokens, &L.kv));
            break;
        case SKN_MIX_LATENT_ATTN:
            rows = 0;
            in_rows(p.heads * (p.dim + p.rot_dims));
            L.latent = {p.heads, p.dim, p.rot_dims, p.vdim, p.kv_rank, p.mask, p.mask_size, p.scale, c.norm_eps, p.latent_norm, L.rot_freq, p.w_latent, type};
            if (p.kv_from < 0) {
                in_rows(p.kv_rank + p.rot_dims);
                SKN_TRY(skn_kv_create_latent(ctx, 1, p.kv_rank, p.rot_dims, cache_type, c.page_tokens, c.max_tokens, &L.kv));
            } else {
                L.kv = m->layers[p.kv_from].kv;
            }
            m->max_attn = std::max(m->max_attn, (int)skn_latent_prep_floats(L.kv, L.latent));
            m->max_lat = std::max(m->max_lat, (int)skn_latent_lat_floats(L.kv, L.latent));
            break;
        case SKN_MIX_CHANNEL_DELTA:
            in_rows(p.kv_heads * p.dim);
            in_rows(p.kv_heads * p.dim);
            in_rows(p.heads);
            rows += skn_pad_rows(p.rank) + skn_pad_rows(p.rank_gate);
            m->max_cols = std::max(m->max_cols, skn_pad_cols(p.heads * p.dim));  // (the decays)
            L.channel = {p.conv, p.decay_rate};
            L.decay = mat(p.w_decay, p.heads * p.dim, p.rank, p.b_decay);
            L.gate = mat(p.w_gate, L.hd, p.rank_gate);
            m->max_rank = std::max(m->max_rank, std::max(L.decay.k_pad, L.gate.k_pad));
            SKN_TRY(skn_rstate_create_conv(ctx, 1, p.heads, p.kv_heads, p.dim, p.vdim, p.taps, &L.state));
            prompt_cols = 10;
            break;
        default:
            rows += 4 * skn_pad_rows(L.hd) + skn_pad_rows(p.rank);
            L.decay = mat(p.w_decay, L.hd, p.rank, p.b_decay);
            m->max_rank = std::max(m->max_rank, L.decay.k_pad);
            SKN_TRY(skn_rstate_create(ctx, 1, p.heads, p.dim, &L.state));
            prompt_cols = 6;
    }
    L.owns_kv = L.kv && !(p.mixer == SKN_MIX_LATENT_ATTN && p.kv_from >= 0);  // (nothing above fails after a cache was made)
    m->prompt_cols = std::max(m->prompt_cols, prompt_cols);
    const int ff_beside = p.norm2 ? 0 : p.ff;
    L.off_ff = skn_pad_cols(L.hd);
    L.in = {p.w_in, type, rows + skn_pad_rows(ff_beside), m->width_pad, p.b_in};
    L.out = {p.w_out, type, skn_pad_rows(c.width), L.off_ff + skn_pad_cols(ff_beside), p.b_out};
    m->max_out = std::max(m->max_out, std::max(L.out.k_pad, skn_pad_cols(p.ff)));
    m->max_ff = std::max(m->max_ff, skn_pad_cols(p.ff));
    if (p.norm2 && p.ff) {
        L.up = mat(p.w_up, p.ff, c.width);
        L.down = mat(p.w_down, c.width, p.ff);
    }
    if (c.side_dim) {
        L.side_gate = mat(p.side_gate, c.side_dim, c.width);
        L.side_proj = mat(p.side_proj, c.width, c.side_dim);
    }
    if (L.kv) {
        m->max_attn = std::max(m->max_attn, p.heads * L.kv->head_dim);
        m->max_heads = std::max(m->max_heads, (int)p.heads);
    }
    return SKN_OK;
}

}  // namespace

extern "C" {

int skn_hybrid_create(skn_ctx* ctx, const skn_hybrid_config* cfg, const skn_hybrid_weights* w, skn_hybrid** out) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_create: ctx is null");
    SKN_REQUIRE(ctx, cfg && w && out, SKN_ERR_ARG, "skn_hybrid_create: null pointer");
    *out = nullptr;
    SKN_REQUIRE(ctx, cfg->n_layer > 0 && cfg->width > 0 && cfg->vocab > 0 && cfg->max_tokens > 0 && cfg->page_tokens > 0 && cfg->norm_groups > 0, SKN_ERR_ARG,
                "skn_hybrid_create: sizes must be positive");
    SKN_REQUIRE(ctx, cfg->side_dim == 0 || (cfg->side_dim > 0 && cfg->norm_groups == 1 && w->side && ((uintptr_t)w->side & 15) == 0), SKN_ERR_ARG,
                "skn_hybrid_create: a side table of %d elements per layer, %d norm groups", cfg->side_dim, cfg->norm_groups);
    SKN_REQUIRE(ctx, cfg->width % cfg->norm_groups == 0 && cfg->norm_groups <= 256, SKN_ERR_SHAPE,
                "skn_hybrid_create: %d norm groups do not divide width %d (at most 256 groups)", cfg->norm_groups, cfg->width);
    SKN_REQUIRE(ctx, cfg->weight_type == SKN_TYPE_BF16 || cfg->weight_type == SKN_TYPE_F32, SKN_ERR_TYPE,
                "skn_hybrid_create: weights of type %d (BF16 or F32)", cfg->weight_type);
    SKN_REQUIRE(ctx, w->layers && w->embed && w->final_norm && w->head, SKN_ERR_ARG, "skn_hybrid_create: missing weights");
    SKN_REQUIRE(ctx, (((uintptr_t)w->embed | (uintptr_t)w->final_norm | (uintptr_t)w->head) & 15) == 0, SKN_ERR_ARG,
                "skn_hybrid_create: weights must be 16-byte aligned");
    for (int l = 0; l < cfg->n_layer; l++) SKN_TRY(check_layer(ctx, *cfg, w->layers, l));
    skn_hybrid* m = new (std::nothrow) skn_hybrid();
    SKN_REQUIRE(ctx, m != nullptr, SKN_ERR_OOM, "skn_hybrid_create: host allocation failed");
    m->cfg = *cfg;
    m->embed = w->embed;
    m->final_norm = w->final_norm;
    m->side = cfg->side_dim ? w->side : nullptr;
    m->side_pad = skn_pad_cols(cfg->side_dim);
    m->width_pad = skn_pad_cols(cfg->width);
    m->head = {w->head, cfg->weight_type, skn_pad_rows(cfg->vocab), m->width_pad, nullptr};
    m->layers.resize(cfg->n_layer);
    int rc = SKN_OK;
    for (int l = 0; l < cfg->n_layer && rc == SKN_OK; l++) {
        m->layers[l].p = w->layers[l];
        rc = build_layer(ctx, m, l);
    }
    auto A = [&](auto** p, size_t floats) {
        if (rc == SKN_OK) rc = dev_alloc(ctx, m, p, floats * 4);
    };
    A(&m->x, m->width_pad);
    A(&m->x2, m->width_pad);
    A(&m->sy, m->width_pad);
    A(&m->sg, m->side_pad);
    A(&m->cols, kStepCols * (size_t)m->max_cols);
    A(&m->mix, m->max_cols);
    A(&m->mid, m->max_ff);
    A(&m->rank, m->max_rank);
    A(&m->rank2, m->max_rank);
    A(&m->qprep, m->max_attn);
    A(&m->logits, skn_pad_cols(cfg->vocab));
    A(&m->opart, 16 * (size_t)m->max_attn);
    A(&m->ml, 32 * (size_t)m->max_heads);
    const int pairs = (cfg->width + 1) / 2;
    A(&m->inv_freq, 2 * (size_t)pairs);
    if (rc == SKN_OK) rc = skn_stepper_create(ctx, &m->step, cfg->max_tokens);
    if (rc == SKN_OK) {
        std::vector<double> f(pairs);
        for (int i = 0; i < pairs; i++) f[i] = pow(10000.0, -2.0 * i / cfg->width);
        rc = skn_upload(ctx, m->inv_freq, f.data(), f.size() * sizeof(double));
    }
    if (rc != SKN_OK) {
        skn_hybrid_free(ctx, m);
        return rc;
    }
    *out = m;
    return SKN_OK;
}

int skn_hybrid_free(skn_ctx* ctx, skn_hybrid* m) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_free: ctx is null");
    if (!m) return SKN_OK;
    (void)hipStreamSynchronize(ctx->stream);
    skn_stepper_free(&m->step);
    for (Layer& L : m->layers) {
        if (L.owns_kv) skn_kv_free(ctx, L.kv);
        if (L.state) skn_rstate_free(ctx, L.state);
    }
    for (void* p : m->owned) (void)hipFree(p);
    if (m->latent_ws.mem) (void)hipFree(m->latent_ws.mem);
    delete m;
    return SKN_OK;
}

int skn_hybrid_reset(skn_ctx* ctx, skn_hybrid* m) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_reset: ctx is null");
    SKN_REQUIRE(ctx, m != nullptr, SKN_ERR_ARG, "skn_hybrid_reset: model is null");
    for (Layer& L : m->layers) {
        if (L.owns_kv) SKN_TRY(skn_kv_reset(ctx, L.kv, 0));
        if (L.state) SKN_TRY(skn_rstate_reset(ctx, L.state, 0));
    }
    m->pos = 0;
    return SKN_OK;
}

int skn_hybrid_prefill(skn_ctx* ctx, skn_hybrid* m, const int32_t* tokens_host, int n_tokens, int32_t* next_token_host) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_prefill: ctx is null");
    SKN_REQUIRE(ctx, m && tokens_host, SKN_ERR_ARG, "skn_hybrid_prefill: null pointer");
    SKN_REQUIRE(ctx, n_tokens > 0, SKN_ERR_ARG, "skn_hybrid_prefill: the prompt is empty");
    SKN_TRY(check_tokens(ctx, m, tokens_host, n_tokens));
    int last = 0;
    SKN_TRY(run_prompt(ctx, m, tokens_host, n_tokens, nullptr, 0, nullptr, &last));
    skn_matvec_src norm;
    norm.mode = SKN_XSRC_GROUP_NORM;
    norm.x0 = m->px + (size_t)(last - 1) * m->width_pad;
    norm.k0 = m->cfg.width;
    norm.groups = m->cfg.norm_groups;
    norm.eps = m->cfg.norm_eps;
    norm.norm_w = m->final_norm;
    skn_dense_out lg;
    add_seg(lg, 0, m->cfg.vocab, SKN_OP_NONE, m->logits, skn_pad_cols(m->cfg.vocab), SKN_TYPE_F32);
    SKN_TRY(skn_dense_matvec(ctx, m->head, norm, lg));
    SKN_TRY(skn_stepper_pick(ctx, &m->step, m->logits, m->cfg.vocab, 0));
    int32_t next = 0;
    SKN_HIP(ctx, hipMemcpyAsync(&next, m->step.tokens_out, sizeof(int32_t), hipMemcpyDeviceToHost, ctx->stream));
    SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    if (next_token_host) *next_token_host = next;
    return SKN_OK;
}

int skn_hybrid_decode(skn_ctx* ctx, skn_hybrid* m, int32_t first_token, int n_steps, int32_t* tokens_out_host) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_decode: ctx is null");
    SKN_REQUIRE(ctx, m != nullptr, SKN_ERR_ARG, "skn_hybrid_decode: model is null");
    SKN_REQUIRE(ctx, n_steps >= 0, SKN_ERR_ARG, "skn_hybrid_decode: negative step count");
    if (n_steps == 0) return SKN_OK;
    SKN_REQUIRE(ctx, tokens_out_host != nullptr, SKN_ERR_ARG, "skn_hybrid_decode: tokens_out is null");
    SKN_TRY(check_tokens(ctx, m, &first_token, 1));
    SKN_REQUIRE(ctx, m->pos + n_steps <= m->cfg.max_tokens, SKN_ERR_POOL, "sequence is full (%d tokens, capacity %d)", m->pos + n_steps, m->cfg.max_tokens);
    SKN_REQUIRE(ctx, !ctx->prof_on || ctx->opt_llama_graph == 0, SKN_ERR_STATE,
                "skn_hybrid_decode: not available while per-launch timing is on (except with llama.graph = 0)");
    return run_steps(ctx, m, first_token, n_steps, tokens_out_host);
}

int skn_hybrid_extend(skn_ctx* ctx, skn_hybrid* m, const int32_t* tokens_host, int n_tokens, const int32_t* want_host, int n_want, float* logits_host) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_extend: ctx is null");
    SKN_REQUIRE(ctx, m && tokens_host, SKN_ERR_ARG, "skn_hybrid_extend: null pointer");
    SKN_REQUIRE(ctx, n_tokens > 0 && n_want >= 0 && (n_want == 0 || (want_host && logits_host)), SKN_ERR_ARG, "skn_hybrid_extend: bad arguments");
    SKN_TRY(check_tokens(ctx, m, tokens_host, n_tokens));
    for (int i = 0; i < n_want; i++)
        SKN_REQUIRE(ctx, want_host[i] >= 0 && want_host[i] < n_tokens && (i == 0 || want_host[i] >= want_host[i - 1]), SKN_ERR_RANGE,
                    "skn_hybrid_extend: wanted row %d of %d (ascending)", want_host[i], n_tokens);
    if (n_tokens == 1) {  // the decode step
        SKN_REQUIRE(ctx, !ctx->prof_on || ctx->opt_llama_graph == 0, SKN_ERR_STATE, "skn_hybrid_extend: not available while per-launch timing is on");
        int32_t next = 0;
        SKN_TRY(run_steps(ctx, m, tokens_host[0], 1, &next));
        for (int i = 0; i < n_want; i++) SKN_TRY(skn_download(ctx, logits_host + (size_t)i * m->cfg.vocab, m->logits, (size_t)m->cfg.vocab * sizeof(float)));
        return SKN_OK;
    }
    int last = 0;
    SKN_TRY(run_prompt(ctx, m, tokens_host, n_tokens, want_host, n_want, logits_host, &last));
    SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    return SKN_OK;
}

int skn_hybrid_logits(skn_ctx* ctx, skn_hybrid* m, const float** logits_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_logits: ctx is null");
    SKN_REQUIRE(ctx, m && logits_dev, SKN_ERR_ARG, "skn_hybrid_logits: null pointer");
    *logits_dev = m->logits;
    return SKN_OK;
}

}  // extern "C"
