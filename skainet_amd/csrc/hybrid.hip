// Decoder over a list of layers that differ from each other: every entry names its mixer -- attention over a shared
// key/value cache, or the generalized delta rule on a recurrent state -- with its own sizes, and a feed-forward or none.
// The two sublayers of a layer run in parallel on one norm:
//
//   h = groupnorm(x);   x += residual_mult * (mixer(h) + Wdown . xielu(Wup h))
//
// with the residual stream in fp32.  What reads h is one stacked matrix and what adds to x is one matrix whose columns are
// the mixer's outputs followed by the feed-forward's, so a layer is, per decode step, three launches: [norm + input projections +
// their activations + key to the cache], mixer, [output projections + residual]; a prompt takes the same products as
// GEMMs with the same epilogues, and the row-wise parts between them.
// Weights are bf16 or fp32; with fp32 weights every operand, the cached keys included, is fp32.
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

struct Layer {
    skn_hybrid_layer p;
    skn_dense_mat in, out, decay;
    int hd = 0, gd = 0, off_ff = 0;  // mixer output columns, key columns, first feed-forward column of `out`
    skn_shared_attn attn;
    skn_kv* kv = nullptr;
    skn_rstate* state = nullptr;
};

}  // namespace

struct skn_hybrid {
    skn_hybrid_config cfg;
    std::vector<Layer> layers;
    skn_dense_mat head;
    const void* embed = nullptr;
    const float* final_norm = nullptr;
    skn_stepper step;
    int pos = 0;
    int width_pad = 0, max_cols = 0, max_out = 0, max_ff = 0, max_rank = 0, max_attn = 0, max_heads = 0;
    double* inv_freq = nullptr;
    // decode-step buffers
    float *x = nullptr, *cols = nullptr, *mix = nullptr, *mid = nullptr, *rank = nullptr, *logits = nullptr, *opart = nullptr, *ml = nullptr;
    // prompt buffers (grown to the longest slice seen)
    int cap = 0;
    float *px = nullptr, *pcols = nullptr, *pq = nullptr, *ppack = nullptr, *plogits = nullptr;
    void *ph = nullptr, *pa = nullptr, *prank = nullptr, *pwant_h = nullptr;
    int32_t *ptok = nullptr, *pwant = nullptr;
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
    dev_release(m, &m->px); dev_release(m, &m->pcols); dev_release(m, &m->pq); dev_release(m, &m->ppack);
    dev_release(m, &m->ph); dev_release(m, &m->pa); dev_release(m, &m->prank); dev_release(m, &m->ptok);
    const size_t es = elem_bytes(m), t = T;
    size_t pack = 0;
    for (const Layer& L : m->layers)
        if (L.state) pack = std::max(pack, skn_delta_pack_floats(L.state, T));
    SKN_TRY(dev_alloc(ctx, m, &m->px, t * m->width_pad * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->pcols, 6 * t * m->max_cols * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->pq, t * m->max_attn * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->ppack, pack * 4));
    SKN_TRY(dev_alloc(ctx, m, &m->ph, t * m->width_pad * es));
    SKN_TRY(dev_alloc(ctx, m, &m->pa, t * m->max_out * es));
    SKN_TRY(dev_alloc(ctx, m, &m->prank, t * m->max_rank * es));
    SKN_TRY(dev_alloc(ctx, m, &m->ptok, t * sizeof(int32_t)));
    m->cap = T;
    return SKN_OK;
}

void add_seg(skn_dense_out& o, int row0, int rows, int op, void* out, int ldo, int type, float p0 = 0.f, float p1 = 0.f) {
    o.seg[o.nseg++] = {row0, rows, op, p0, p1, out, ldo, type};
}

// The rows of a layer's input matrix, in order: attention q, k; delta rule r, k, v, g, a, w1; then the feed-forward.
// cols: where the fp32 ones go (segment i at cols + i * col_stride, rows of ldc); the low-rank ones to `rank`, the
// feed-forward's to `mid`, both of mid_type.
skn_dense_out input_segments(const Layer& L, float* cols, int64_t col_stride, int ldc, void* rank, int ldr, void* mid, int ldm, int mid_type) {
    skn_dense_out o;
    int row = 0;
    auto put = [&](int rows, int op, void* out, int ld, int type, float p0 = 0.f, float p1 = 0.f) {
        add_seg(o, row, rows, op, out, ld, type, p0, p1);
        row += skn_pad_rows(rows);
    };
    if (L.kv) {
        put(L.hd, SKN_OP_NONE, cols, ldc, SKN_TYPE_F32);
        put(L.gd, SKN_OP_NONE, cols + col_stride, ldc, SKN_TYPE_F32);
    } else {
        for (int i = 0; i < 3; i++) put(L.hd, SKN_OP_NONE, cols + i * col_stride, ldc, SKN_TYPE_F32);
        for (int i = 3; i < 5; i++) put(L.hd, SKN_OP_SIGMOID, cols + i * col_stride, ldc, SKN_TYPE_F32);
        put(L.p.rank, SKN_OP_TANH, rank, ldr, mid_type);
    }
    if (L.p.ff) put(L.p.ff, SKN_OP_XIELU, mid, ldm, mid_type, L.p.act_pos, L.p.act_neg);
    return o;
}

// ---- decode -----------------------------------------------------------------------------------------------------------

int decode_step(skn_ctx* ctx, skn_hybrid* m, int max_ctx) {
    const skn_hybrid_config& c = m->cfg;
    SKN_TRY(skn_embed_sinusoid_rows(ctx, m->embed, c.weight_type, m->width_pad, m->step.state, m->step.state + 1, m->inv_freq, 1, c.width, m->x, m->width_pad));
    skn_matvec_src norm;
    norm.mode = SKN_XSRC_GROUP_NORM;
    norm.x0 = m->x;
    norm.k0 = c.width;
    norm.groups = c.norm_groups;
    norm.eps = c.norm_eps;
    for (Layer& L : m->layers) {
        skn_dense_out in = input_segments(L, m->cols, m->max_cols, m->max_cols, m->rank, m->max_rank, m->mid, m->max_ff, SKN_TYPE_F32);
        if (L.kv) {
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
        norm.norm_w = L.p.norm;
        SKN_TRY(skn_dense_matvec(ctx, L.in, norm, in));
        skn_matvec_src src;
        src.x0 = m->mix;
        src.k0 = L.hd;
        if (L.p.ff) {
            src.x1 = m->mid;
            src.off1 = L.off_ff;
            src.k1 = L.p.ff;
        }
        if (L.kv) {
            const int splits = skn_shared_attn_splits(ctx, L.kv, L.attn.n_head, max_ctx);
            SKN_TRY(skn_shared_attn_step(ctx, L.kv, 0, L.attn, m->cols, m->cols + m->max_cols, m->step.state, splits, m->opart, m->ml, m->mix));
            if (splits > 1) {
                src.mode = SKN_XSRC_MERGE;
                src.x0 = m->opart;
                src.ml = m->ml;
                src.splits = splits;
                src.heads = L.attn.n_head;
                src.dim = L.kv->dim;
                src.dim_pad = L.kv->head_dim;
            }
        } else {
            skn_delta_step d;
            const int64_t s = m->max_cols;
            d.r = m->cols, d.k = m->cols + s, d.v = m->cols + 2 * s, d.g = m->cols + 3 * s, d.a = m->cols + 4 * s;
            d.t = m->rank;
            d.w2 = L.decay.w;
            d.w2_type = L.decay.type;
            d.rank = L.p.rank;
            d.rank_pad = L.decay.k_pad;
            d.b2 = L.decay.bias;
            d.norm = L.p.o_norm;
            d.eps = c.norm_eps;
            d.y = m->mix;
            SKN_TRY(skn_delta_step_launch(ctx, L.state, 0, d));
        }
        skn_dense_out out;
        out.resid = m->x;
        out.ldr = m->width_pad;
        out.resid_rows = c.width;
        out.mult = c.residual_mult;
        SKN_TRY(skn_dense_matvec(ctx, L.out, src, out));
    }
    norm.norm_w = m->final_norm;
    skn_dense_out lg;
    add_seg(lg, 0, c.vocab, SKN_OP_NONE, m->logits, skn_pad_cols(c.vocab), SKN_TYPE_F32);
    SKN_TRY(skn_dense_matvec(ctx, m->head, norm, lg));
    return skn_stepper_pick(ctx, &m->step, m->logits, c.vocab, 1);
}

int run_steps(skn_ctx* ctx, skn_hybrid* m, int first_token, int n_steps, int32_t* tokens_out_host) {
    for (Layer& L : m->layers)
        if (L.kv) SKN_TRY(skn_kv_reserve(ctx, L.kv, 0, m->pos + n_steps));
    // the step is captured for contexts up to a power of two (the attention's split counts), again when a run passes it
    int max_ctx = 128;
    while (max_ctx < m->pos + n_steps) max_ctx *= 2;
    SKN_TRY(skn_stepper_run(ctx, &m->step, first_token, m->pos, n_steps, max_ctx, [&]() { return decode_step(ctx, m, max_ctx); }, tokens_out_host));
    m->pos += n_steps;
    for (Layer& L : m->layers)
        if (L.kv) L.kv->len[0] = m->pos;
    return SKN_OK;
}

// ---- prompts ----------------------------------------------------------------------------------------------------------

// n tokens (device ids in m->ptok) through all layers; the residual rows are left in m->px
int run_slice(skn_ctx* ctx, skn_hybrid* m, int n) {
    const skn_hybrid_config& c = m->cfg;
    const int pos0 = m->pos, type = c.weight_type;
    for (Layer& L : m->layers)
        if (L.kv) SKN_TRY(skn_kv_reserve(ctx, L.kv, 0, pos0 + n));
    SKN_TRY(skn_stepper_set(ctx, &m->step, 0, pos0));
    SKN_TRY(skn_embed_sinusoid_rows(ctx, m->embed, type, m->width_pad, m->ptok, m->step.state + 1, m->inv_freq, n, c.width, m->px, m->width_pad));
    const int64_t stride = (int64_t)n * m->max_cols;
    auto col = [&](int i) { return m->pcols + i * stride; };
    for (Layer& L : m->layers) {
        SKN_TRY(skn_group_norm_rows(ctx, m->px, m->width_pad, nullptr, L.p.norm, n, c.width, c.norm_groups, c.norm_eps, m->ph, m->width_pad, type));
        const int lda = L.out.k_pad;  // the output product's activations: mixer columns, then the feed-forward's
        void* mid = (uint8_t*)m->pa + (size_t)L.off_ff * elem_bytes(m);
        const skn_dense_out in = input_segments(L, m->pcols, stride, m->max_cols, m->prank, L.kv ? 0 : L.decay.k_pad, mid, lda, type);
        SKN_TRY(skn_dense_gemm(ctx, L.in, m->ph, m->width_pad, n, in));
        if (L.kv) {
            SKN_TRY(skn_shared_prep_rows(ctx, L.kv, 0, L.attn, col(0), m->max_cols, col(1), m->max_cols, n, pos0, m->pq));
            SKN_TRY(skn_shared_attn_rows(ctx, L.kv, 0, L.attn, m->pq, n, pos0, m->pa, lda, type));
            L.kv->len[0] = pos0 + n;
        } else {
            skn_dense_out w;
            add_seg(w, 0, L.hd, SKN_OP_DECAY, col(5), m->max_cols, SKN_TYPE_F32);
            SKN_TRY(skn_dense_gemm(ctx, L.decay, m->prank, L.decay.k_pad, n, w));
            float* o = col(5);  // (the decays are packed before the scan writes its outputs over them)
            SKN_TRY(skn_delta_rows(ctx, L.state, 0, col(0), col(1), col(2), col(5), col(4), m->max_cols, n, m->ppack, o));
            SKN_TRY(skn_delta_gate_rows(ctx, o, col(3), m->max_cols, L.p.o_norm, n, L.p.heads, L.p.dim, c.norm_eps, m->pa, lda, type));
        }
        skn_dense_out out;
        out.resid = m->px;
        out.ldr = m->width_pad;
        out.resid_rows = c.width;
        out.mult = c.residual_mult;
        SKN_TRY(skn_dense_gemm(ctx, L.out, m->pa, lda, n, out));
    }
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

int check_layer(skn_ctx* ctx, const skn_hybrid_layer& p, int l) {
    const bool attn = p.mixer == SKN_MIX_SHARED_ATTN, delta = p.mixer == SKN_MIX_GENERAL_DELTA;
    SKN_REQUIRE(ctx, attn || delta, SKN_ERR_TYPE, "skn_hybrid_create: layer %d has an unknown mixer (%d)", l, p.mixer);
    SKN_REQUIRE(ctx, p.heads > 0 && p.dim > 0 && p.dim <= 256 && p.ff >= 0, SKN_ERR_SHAPE, "skn_hybrid_create: layer %d: %d heads of %d (at most 256)", l,
                p.heads, p.dim);
    SKN_REQUIRE(ctx, p.norm && p.w_in && p.b_in && p.w_out && p.b_out, SKN_ERR_ARG, "skn_hybrid_create: layer %d has a null weight", l);
    SKN_REQUIRE(ctx, (((uintptr_t)p.w_in | (uintptr_t)p.w_out | (uintptr_t)p.norm | (uintptr_t)p.b_in | (uintptr_t)p.b_out | (uintptr_t)p.w_decay) & 15) == 0,
                SKN_ERR_ARG, "skn_hybrid_create: the weights of layer %d must be 16-byte aligned", l);
    if (attn) {
        SKN_REQUIRE(ctx, p.kv_heads > 0 && p.heads % p.kv_heads == 0, SKN_ERR_SHAPE, "skn_hybrid_create: layer %d: kv_heads (%d) must divide heads (%d)", l,
                    p.kv_heads, p.heads);
        SKN_REQUIRE(ctx, p.q_norm && p.k_norm && (p.temp_coef == 0.f || p.temp_every > 0.f), SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad attention parameters", l);
    } else {
        SKN_REQUIRE(ctx, p.rank > 0 && p.w_decay && p.b_decay && p.o_norm, SKN_ERR_ARG, "skn_hybrid_create: layer %d: bad delta rule parameters", l);
    }
    return SKN_OK;
}

int build_layer(skn_ctx* ctx, skn_hybrid* m, Layer& L) {
    const skn_hybrid_config& c = m->cfg;
    const skn_hybrid_layer& p = L.p;
    L.hd = p.heads * p.dim;
    L.gd = p.mixer == SKN_MIX_SHARED_ATTN ? p.kv_heads * p.dim : 0;
    L.off_ff = skn_pad_cols(L.hd);
    const int rows = p.mixer == SKN_MIX_SHARED_ATTN ? skn_pad_rows(L.hd) + skn_pad_rows(L.gd) : 5 * skn_pad_rows(L.hd) + skn_pad_rows(p.rank);
    L.in = {p.w_in, c.weight_type, rows + skn_pad_rows(p.ff), m->width_pad, p.b_in};
    L.out = {p.w_out, c.weight_type, skn_pad_rows(c.width), L.off_ff + skn_pad_cols(p.ff), p.b_out};
    m->max_cols = std::max(m->max_cols, skn_pad_cols(L.hd));
    m->max_out = std::max(m->max_out, L.out.k_pad);
    m->max_ff = std::max(m->max_ff, skn_pad_cols(p.ff));
    if (p.mixer == SKN_MIX_SHARED_ATTN) {
        L.attn = {p.heads, p.scale, p.temp_coef, p.temp_every, c.norm_eps, p.q_norm, p.k_norm};
        SKN_TRY(skn_kv_create_shared(ctx, 1, p.kv_heads, p.dim, c.weight_type == SKN_TYPE_F32 ? SKN_TYPE_F32 : SKN_TYPE_F16, c.page_tokens, c.max_tokens, &L.kv));
        m->max_attn = std::max(m->max_attn, p.heads * L.kv->head_dim);
        m->max_heads = std::max(m->max_heads, (int)p.heads);
    } else {
        L.decay = {p.w_decay, c.weight_type, skn_pad_rows(L.hd), skn_pad_cols(p.rank), p.b_decay};
        m->max_rank = std::max(m->max_rank, L.decay.k_pad);
        SKN_TRY(skn_rstate_create(ctx, 1, p.heads, p.dim, &L.state));
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
    SKN_REQUIRE(ctx, cfg->width % cfg->norm_groups == 0 && cfg->norm_groups <= 256, SKN_ERR_SHAPE,
                "skn_hybrid_create: %d norm groups do not divide width %d (at most 256 groups)", cfg->norm_groups, cfg->width);
    SKN_REQUIRE(ctx, cfg->weight_type == SKN_TYPE_BF16 || cfg->weight_type == SKN_TYPE_F32, SKN_ERR_TYPE,
                "skn_hybrid_create: weights of type %d (BF16 or F32)", cfg->weight_type);
    SKN_REQUIRE(ctx, w->layers && w->embed && w->final_norm && w->head, SKN_ERR_ARG, "skn_hybrid_create: missing weights");
    SKN_REQUIRE(ctx, (((uintptr_t)w->embed | (uintptr_t)w->final_norm | (uintptr_t)w->head) & 15) == 0, SKN_ERR_ARG,
                "skn_hybrid_create: weights must be 16-byte aligned");
    for (int l = 0; l < cfg->n_layer; l++) SKN_TRY(check_layer(ctx, w->layers[l], l));
    skn_hybrid* m = new (std::nothrow) skn_hybrid();
    SKN_REQUIRE(ctx, m != nullptr, SKN_ERR_OOM, "skn_hybrid_create: host allocation failed");
    m->cfg = *cfg;
    m->embed = w->embed;
    m->final_norm = w->final_norm;
    m->width_pad = skn_pad_cols(cfg->width);
    m->head = {w->head, cfg->weight_type, skn_pad_rows(cfg->vocab), m->width_pad, nullptr};
    m->layers.resize(cfg->n_layer);
    int rc = SKN_OK;
    for (int l = 0; l < cfg->n_layer && rc == SKN_OK; l++) {
        m->layers[l].p = w->layers[l];
        rc = build_layer(ctx, m, m->layers[l]);
    }
    auto A = [&](auto** p, size_t floats) {
        if (rc == SKN_OK) rc = dev_alloc(ctx, m, p, floats * 4);
    };
    A(&m->x, m->width_pad);
    A(&m->cols, 5 * (size_t)m->max_cols);
    A(&m->mix, m->max_cols);
    A(&m->mid, m->max_ff);
    A(&m->rank, m->max_rank);
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
        if (L.kv) skn_kv_free(ctx, L.kv);
        if (L.state) skn_rstate_free(ctx, L.state);
    }
    for (void* p : m->owned) (void)hipFree(p);
    delete m;
    return SKN_OK;
}

int skn_hybrid_reset(skn_ctx* ctx, skn_hybrid* m) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_hybrid_reset: ctx is null");
    SKN_REQUIRE(ctx, m != nullptr, SKN_ERR_ARG, "skn_hybrid_reset: model is null");
    for (Layer& L : m->layers) {
        if (L.kv) SKN_TRY(skn_kv_reset(ctx, L.kv, 0));
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
