// Attention over a range of the cache (all, a window, or a chunk) with separate keys and values: per head, q and k are divided by
// their root mean square and rotated in part; scores may be capped, the softmax may have a sink, the output may be gated.
// A decode step is one launch (the prologue of attention_stream.h); a prompt is prepared row by row and attended to on the matrix
// cores (csrc/attention_prefill.hip) or, from fp32 caches and heads beyond 128 elements, by the streaming kernel.
#include "attention_stream.h"

#include <algorithm>

namespace {

constexpr int kMaxSplits = 16;  // what the merge in the output projection's staging is fed at most

// one workgroup per row, a wavefront per head at a time: q heads to q_prep, k and v heads to the cache
template <typename E>
__global__ __launch_bounds__(256) void ranged_prep_kernel(const skn_ranged_attn p, const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk,
                                                          const float* __restrict__ v, int ldv, E* __restrict__ k_pool, E* __restrict__ v_pool,
                                                          const int32_t* __restrict__ table, int page_tokens, int kv_heads, int kdim, int vdim, int width,
                                                          int pos0, float* __restrict__ q_prep) {
    __shared__ float sn[128], cs[128], x[4][256];
    const int row = blockIdx.x, pos = pos0 + row, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, half = p.rot_dims >> 1;
    if (tid < half) skn_rope_sincos_freq(pos, p.rot_freq[tid], &sn[tid], &cs[tid]);
    const int page = table[pos / page_tokens], slot = pos % page_tokens, heads = p.n_head + kv_heads;
    __syncthreads();
    for (int h = wave; h < heads; h += 4) {
        const bool is_q = h < p.n_head;
        const float* src = is_q ? q + (int64_t)row * ldq + h * kdim : k + (int64_t)row * ldk + (h - p.n_head) * kdim;
        const float* norm = is_q ? p.q_norm : p.k_norm;
        float r[4], ss = 0.f;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int e = lane + 64 * j;
            r[j] = e < kdim ? src[e] : 0.f;
            ss = fmaf(r[j], r[j], ss);
        }
        const float f = norm ? 1.0f / sqrtf(wave_sum(ss) / (float)kdim + p.eps) : 1.f;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int e = lane + 64 * j;
            x[wave][e] = r[j] * f * (norm && e < kdim ? norm[e] : 1.f);
        }
        // (a wavefront's own part of LDS, whose accesses take effect in order)
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int e = lane + 64 * j;
            float y = x[wave][e];
            if (e < half) y = y * cs[e] - x[wave][e + half] * sn[e];
            else if (e < p.rot_dims) y = y * cs[e - half] + x[wave][e - half] * sn[e - half];
            if (is_q && e < width) q_prep[((int64_t)row * p.n_head + h) * width + e] = y;
            else if (!is_q && e < kdim) store_cached(k_pool + (((int64_t)page * kv_heads + (h - p.n_head)) * page_tokens + slot) * width + e, y);
        }
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
    }
    for (int e = tid; e < kv_heads * vdim; e += 256) {
        const int h = e / vdim, d = e - h * vdim;
        store_cached(v_pool + (((int64_t)page * kv_heads + h) * page_tokens + slot) * width + d, v[(int64_t)row * ldv + e]);
    }
}

template <typename E, int KIND>
int launch_stream(skn_ctx* ctx, const skn_kv* kv, const StreamArgs& a, int rows) {
    const dim3 grid(a.n_splits, a.n_head, rows), block(stream_threads<KIND>());
    if (kv->head_dim == 64) skn_launch(ctx, stream_attn_kernel<E, 8, 1, KIND>, grid, block, 0, a);
    else if (kv->head_dim == 128) skn_launch(ctx, stream_attn_kernel<E, 16, 1, KIND>, grid, block, 0, a);
    else skn_launch(ctx, stream_attn_kernel<E, 32, 1, KIND>, grid, block, 0, a);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

StreamArgs ranged_args(const skn_kv* kv, int seq, const skn_ranged_attn& p) {
    StreamArgs a = stream_args(kv, seq, p.n_head);
    a.scale = p.scale;
    a.softcap = p.softcap;
    a.range.kind = p.mask;
    a.range.size = p.mask_size;
    a.sink = p.sink;
    return a;
}

int check(skn_ctx* ctx, const skn_kv* kv, const skn_ranged_attn& p) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_RANGED, SKN_ERR_STATE, "ranged attention: not a ranged cache");
    SKN_REQUIRE(ctx, p.n_head > 0 && p.n_head % kv->n_head == 0, SKN_ERR_SHAPE, "ranged attention: %d query heads over %d cached heads", p.n_head, kv->n_head);
    SKN_REQUIRE(ctx, p.rot_dims >= 0 && p.rot_dims % 2 == 0 && p.rot_dims <= kv->dim && (p.rot_dims == 0 || p.rot_freq), SKN_ERR_ARG,
                "ranged attention: %d rotated elements of %d", p.rot_dims, kv->dim);
    SKN_REQUIRE(ctx, p.mask == SKN_MASK_CAUSAL || ((p.mask == SKN_MASK_WINDOW || p.mask == SKN_MASK_CHUNK) && p.mask_size > 0), SKN_ERR_ARG,
                "ranged attention: mask %d of %d tokens", p.mask, p.mask_size);
    return SKN_OK;
}

}  // namespace

int skn_range_longest(const skn_range& r, int max_ctx) { return r.kind == SKN_MASK_CAUSAL ? max_ctx : std::min(max_ctx, r.size); }

// As skn_shared_attn_splits: a power of two, so that a workgroup has at least a round of requests; streams: rows of a workgroup and round.
int skn_ranged_splits(skn_ctx* ctx, int n_head, int streams, const skn_range& r, int max_ctx) {
    const int most = n_head * 8 <= ctx->compute_units / 2 ? kMaxSplits : 8, longest = skn_range_longest(r, max_ctx);
    int n = 1;
    while (n < most && n * streams < longest) n *= 2;
    return n;
}

int skn_ranged_prep_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q, int ldq, const float* k, int ldk, const float* v,
                         int ldv, int n, int pos0, float* q_prep) {
    SKN_TRY(check(ctx, kv, p));
    const int32_t* table = kv->page_table_dev + (size_t)seq * kv->pages_per_seq;
    if (kv->elem_type == SKN_TYPE_F32)
        skn_launch(ctx, ranged_prep_kernel<float>, dim3(n), dim3(256), 0, p, q, ldq, k, ldk, v, ldv, (float*)kv->k_pool, (float*)kv->v_pool, table,
                   kv->page_tokens, kv->n_head, kv->dim, kv->vdim, kv->head_dim, pos0, q_prep);
    else
        skn_launch(ctx, ranged_prep_kernel<uint16_t>, dim3(n), dim3(256), 0, p, q, ldq, k, ldk, v, ldv, kv->k_pool, kv->v_pool, table, kv->page_tokens,
                   kv->n_head, kv->dim, kv->vdim, kv->head_dim, pos0, q_prep);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_ranged_attn_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q_prep, int n, int pos0, const float* gate, int ldg,
                         void* out, int ldo, int out_type) {
    SKN_TRY(check(ctx, kv, p));
    if (skn_ranged_prefill_fits(kv)) {
        skn_prefill_ranged r;
        r.range.kind = p.mask;
        r.range.size = p.mask_size;
        r.scale = p.scale;
        r.softcap = p.softcap;
        r.sink = p.sink;
        r.vdim = kv->vdim;
        r.gate = gate;
        r.ldg = ldg;
        r.out = out;
        r.ldo = ldo;
        r.out_type = out_type;
        return skn_ranged_prefill_launch(ctx, kv, seq, q_prep, n, pos0, p.n_head, r);
    }
    StreamArgs a = ranged_args(kv, seq, p);
    a.ldo = ldo;
    a.out_type = out_type;
    a.ldg = ldg;
    for (int z = 0; z < n; z += 32768) {  // (grid limit)
        a.q_prep = q_prep + (int64_t)z * p.n_head * kv->head_dim;
        a.first_ctx = pos0 + z + 1;
        a.gate = gate ? gate + (int64_t)z * ldg : nullptr;
        a.out = (uint8_t*)out + (int64_t)z * ldo * (out_type == SKN_TYPE_F32 ? 4 : 2);
        const int rows = std::min(n - z, 32768);
        SKN_TRY((kv->elem_type == SKN_TYPE_F32 ? launch_stream<float, kStreamRows>(ctx, kv, a, rows) : launch_stream<uint16_t, kStreamRows>(ctx, kv, a, rows)));
    }
    return SKN_OK;
}

int skn_ranged_attn_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q, const float* k, const float* v, const float* gate,
                         const int32_t* state_dev, int n_splits, float* opart, float* ml, float* out) {
    SKN_TRY(check(ctx, kv, p));
    SKN_REQUIRE(ctx, n_splits >= 1 && n_splits <= kMaxSplits && (n_splits == 1 ? out != nullptr : opart && ml), SKN_ERR_ARG,
                "ranged attention: %d splits without their buffers", n_splits);
    StreamArgs a = ranged_args(kv, seq, p);
    a.q = q;
    a.k = k;
    a.v = v;
    a.q_norm = p.q_norm;
    a.k_norm = p.k_norm;
    a.freq = p.rot_freq;
    a.rot_dims = p.rot_dims;
    a.eps = p.eps;
    a.gate = gate;
    a.state = state_dev;
    a.n_splits = n_splits;
    a.opart = opart;
    a.ml = ml;
    a.out = out;
    a.out_type = SKN_TYPE_F32;
    return kv->elem_type == SKN_TYPE_F32 ? launch_stream<float, kStreamStep>(ctx, kv, a, 1) : launch_stream<uint16_t, kStreamStep>(ctx, kv, a, 1);
}

extern "C" int skn_attn_ranged(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn* p, const float* q_dev, const float* k_dev, const float* v_dev,
                               const float* gate_dev, int n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_attn_ranged: ctx is null");
    SKN_REQUIRE(ctx, kv && p && q_dev && k_dev && v_dev && out_dev, SKN_ERR_ARG, "skn_attn_ranged: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < kv->n_seq && n > 0, SKN_ERR_RANGE, "skn_attn_ranged: %d tokens of sequence %d of %d", n, seq, kv->n_seq);
    SKN_TRY(check(ctx, kv, *p));
    const int pos0 = kv->len[seq], ldo = p->n_head * kv->vdim;
    SKN_TRY(skn_kv_reserve(ctx, kv, seq, pos0 + n));
    void* scratch = nullptr;
    SKN_HIP(ctx, hipMalloc(&scratch, n == 1 ? 16 : (size_t)n * p->n_head * kv->head_dim * sizeof(float)));
    int rc;
    if (n == 1) {
        const int32_t state[4] = {0, pos0, pos0 + 1, 0};
        rc = skn_upload(ctx, scratch, state, sizeof(state));
        if (rc == SKN_OK) rc = skn_ranged_attn_step(ctx, kv, seq, *p, q_dev, k_dev, v_dev, gate_dev, (const int32_t*)scratch, 1, nullptr, nullptr, out_dev);
    } else {
        rc = skn_ranged_prep_rows(ctx, kv, seq, *p, q_dev, p->n_head * kv->dim, k_dev, kv->n_head * kv->dim, v_dev, kv->n_head * kv->vdim, n, pos0,
                                  (float*)scratch);
        if (rc == SKN_OK) rc = skn_ranged_attn_rows(ctx, kv, seq, *p, (const float*)scratch, n, pos0, gate_dev, ldo, out_dev, ldo, SKN_TYPE_F32);
    }
    if (rc == SKN_OK) rc = skn_kv_advance_len(ctx, kv, seq, n);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(scratch);
    return rc;
}
