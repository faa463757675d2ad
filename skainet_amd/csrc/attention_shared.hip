// Attention whose values are its keys before their norm (one cached row per token and key head), with RMS norm of query
// and key over their whole projections, a query temperature by position and a linear distance bias:
//
//   q' = q / rms(q) * q_norm * (1 + coef ln(floor((p + 1) / every) + 1)),   k' = k / rms(k) * k_norm,   v = k
//   out_i = softmax_j <= i ( scale q'_i . k'_j - slope_h (i - j) ) v_j,      slope_h = 2^(-8 (h + 1) / n_head)
//
// The cache keeps the projected k (fp16 or fp32) and one factor 1 / rms(k) per token: the norm weights of the key go to the
// query side (q' . k' = (q' k_norm) . k / rms(k)), so a row serves as key and as value and is read once for both.  Where the
// query heads alone would fill the device several times over, a workgroup takes two of a group at once.
//
// Token streams as in csrc/attention.hip: a row is spread over head_dim / 8 lanes, the lanes of a row own a private softmax
// stream per query head, nothing is staged and no barrier is met while tokens stream.  A step's launch computes the two
// norms of its own token in its prologue (every workgroup for itself, from L2) while its first rows are on their way.
#include "attention_stream.h"
#include "dense.h"
#include "kv.h"

#include <algorithm>

namespace {

constexpr int kThreads = 1024, kWaves = kThreads / 64;
constexpr int kU = 4;           // rows per stream in flight
constexpr int kMaxSplits = 16;  // what the merge in the output projection's staging is fed at most
__device__ __forceinline__ float query_temperature(int pos, float coef, float every) {
    // (the quotient of two integers below 2^24 does not round up to the next one)
    return coef == 0.f ? 1.f : fmaf(coef, logf(floorf((float)(pos + 1) / every) + 1.0f), 1.0f);
}

struct AttnArgs {
    const void* pool;
    float* key_scale;
    const int32_t* table;  // the sequence's row of the page table
    int page_tokens, pages_per_seq, n_head, kv_heads, dim;
    float inv_page;
    float scale_log2e;
    int n_splits;
    float* opart;
    float* ml;
    void* out;
    int ldo, out_type;
    // rows of a prompt: prepared queries, row z sees first_ctx + z tokens
    const float* q_prep;
    int first_ctx;
    // one token: raw projections and their norms
    const float* q;
    const float* k;
    const float* q_norm;
    const float* k_norm;
    const int32_t* state;
    float eps, temp_coef, temp_every;
};

// the part of the sum of squares of x[0, n) that this thread has, in two steps so that the first can be issued early: one
// float4 per thread, then what is left
__device__ __forceinline__ int whole_quads(const float* x, int n) { return ((uintptr_t)x & 15) == 0 ? n >> 2 : 0; }
__device__ __forceinline__ float4 first_quad(const float* x, int n) {
    return (int)threadIdx.x < whole_quads(x, n) ? reinterpret_cast<const float4*>(x)[threadIdx.x] : make_float4(0.f, 0.f, 0.f, 0.f);
}
__device__ __forceinline__ float sum_squares(const float4& v, const float* x, int n) {
    float a = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    const int n4 = whole_quads(x, n);
    for (int i = threadIdx.x + blockDim.x; i < n4; i += blockDim.x) {
        const float4 w = reinterpret_cast<const float4*>(x)[i];
        a += (w.x * w.x + w.y * w.y) + (w.z * w.z + w.w * w.w);
    }
    for (int i = 4 * n4 + threadIdx.x; i < n; i += blockDim.x) a = fmaf(x[i], x[i], a);
    return a;
}

// sums of a and b over the workgroup; red: two floats per wavefront (a barrier inside)
__device__ __forceinline__ void block_sum2(float& a, float& b, float* red) {
    a = wave_sum(a);
    b = wave_sum(b);
    const int wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    if ((threadIdx.x & 63) == 0) red[wave] = a, red[nw + wave] = b;
    __syncthreads();
    a = b = 0.f;
    for (int i = 0; i < nw; i++) a += red[i], b += red[nw + i];
}

// grid (splits, kv heads x head groups, query rows)
template <typename E, int D, int QG, bool STEP>
__global__ __launch_bounds__(kThreads) void shared_attn_kernel(const AttnArgs p) {
    constexpr int LPT = D / 8, G = 64 / LPT, NS = kWaves * G, U = kU;
    __shared__ float so[kWaves][QG][D];
    __shared__ float sm[kWaves][QG], sl[kWaves][QG];
    __shared__ float red[2 * kWaves];
    __shared__ __align__(16) float qs[STEP ? QG * D : 4];
    const int split = blockIdx.x, row = blockIdx.z;
    const int per_kv = p.n_head / p.kv_heads, n_groups = (per_kv + QG - 1) / QG;
    const int kvh = blockIdx.y / n_groups, h0 = kvh * per_kv + (blockIdx.y % n_groups) * QG, h_end = (kvh + 1) * per_kv;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int c = lane % LPT, g = lane / LPT, stream = wave * G + g;
    // what does not wait for the position is requested first: the token's projections, whose norms are computed while the
    // first cached rows are on their way
    float4 q4, k4;
    float q_elem = 0.f;
    if constexpr (STEP) {
        static_assert(QG * D <= kThreads, "one element of the group's queries per thread");
        q4 = first_quad(p.q, p.n_head * p.dim);
        k4 = first_quad(p.k, p.kv_heads * p.dim);
        const int i = tid / D, d = tid - i * D, h = min(h0 + i, h_end - 1);
        if (tid < QG * D && d < p.dim) q_elem = p.q[h * p.dim + d] * p.q_norm[h * p.dim + d] * p.k_norm[kvh * p.dim + d];
    }
    const int n = STEP ? p.state[2] : p.first_ctx + row;
    const int per = ((n + p.n_splits - 1) / p.n_splits + NS - 1) / NS * NS;
    const int t_begin = split * per, t_end = min(n, t_begin + per);
    const E* pool = (const E*)p.pool;
    // the first 64 page ids ride in a register (lane i holds page i)
    const int my_page = p.table[min(lane, p.pages_per_seq - 1)];

    Row8<E> cur[U], nxt[U];
    float cs_cur[U], cs_nxt[U];
    auto fetch = [&](Row8<E>(&rows)[U], float(&cs)[U], int base) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int t = max(min(base + u * NS + stream, t_end - 1), 0);  // past the end: a valid row, masked below
            const int pi = (int)(((float)t + 0.5f) * p.inv_page), slot = t - pi * p.page_tokens;  // (exact below 2^22 tokens)
            int page = __shfl(my_page, pi & 63, 64);
            if (pi >= 64) page = p.table[pi];
            rows[u].load(pool + (((int64_t)page * p.kv_heads + kvh) * p.page_tokens + slot) * D + c * 8);
            cs[u] = p.key_scale[(int64_t)page * p.page_tokens + slot];
        }
    };
    if (t_begin < t_end) fetch(cur, cs_cur, t_begin);

    float qf[QG][8], fq = p.scale_log2e, newest_scale = 0.f;
    if constexpr (STEP) {
        if (tid < QG * D) qs[tid] = q_elem;  // (the barrier of the sums covers it)
        float sq = sum_squares(q4, p.q, p.n_head * p.dim), sk = sum_squares(k4, p.k, p.kv_heads * p.dim);
        block_sum2(sq, sk, red);
        newest_scale = 1.0f / sqrtf(sk / (float)(p.kv_heads * p.dim) + p.eps);
        fq *= query_temperature(n - 1, p.temp_coef, p.temp_every) / sqrtf(sq / (float)(p.n_head * p.dim) + p.eps);
        if (split == 0 && blockIdx.y == 0 && tid == 0) {  // for the steps to come (this one uses its own)
            const int pi = (n - 1) / p.page_tokens;
            p.key_scale[(int64_t)p.table[pi] * p.page_tokens + (n - 1) - pi * p.page_tokens] = newest_scale;
        }
#pragma unroll
        for (int i = 0; i < QG; i++) {
            const float4 a = *reinterpret_cast<const float4*>(&qs[i * D + c * 8]), b = *reinterpret_cast<const float4*>(&qs[i * D + c * 8 + 4]);
            qf[i][0] = a.x, qf[i][1] = a.y, qf[i][2] = a.z, qf[i][3] = a.w, qf[i][4] = b.x, qf[i][5] = b.y, qf[i][6] = b.z, qf[i][7] = b.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < QG; i++) {
            const float4* qp = reinterpret_cast<const float4*>(p.q_prep + ((int64_t)row * p.n_head + min(h0 + i, h_end - 1)) * D + c * 8);
            const float4 a = qp[0], b = qp[1];
            qf[i][0] = a.x, qf[i][1] = a.y, qf[i][2] = a.z, qf[i][3] = a.w, qf[i][4] = b.x, qf[i][5] = b.y, qf[i][6] = b.z, qf[i][7] = b.w;
        }
    }
    float slope[QG], o[QG][8], m_run[QG], l_run[QG];
#pragma unroll
    for (int i = 0; i < QG; i++) {
        slope[i] = exp2f(-8.0f * (float)(h0 + i + 1) / (float)p.n_head) * kLog2e;
        m_run[i] = -INFINITY;
        l_run[i] = 0.f;
#pragma unroll
        for (int j = 0; j < 8; j++) o[i][j] = 0.f;
    }

    auto absorb = [&](const Row8<E>(&rows)[U], const float(&cs)[U], int base) __attribute__((always_inline)) {
        float sc[QG][U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            float kf[8];
            rows[u].get(kf);
            const int t = base + u * NS + stream;
            const float f = (STEP && t == n - 1 ? newest_scale : cs[u]) * fq;
            const float back = (float)(n - 1 - t);
#pragma unroll
            for (int i = 0; i < QG; i++) {
                float d = 0.f;
#pragma unroll
                for (int j = 0; j < 8; j++) d = fmaf(kf[j], qf[i][j], d);
                d = lane_group_sum<LPT>(d);
                sc[i][u] = t < t_end ? fmaf(d, f, -slope[i] * back) : -INFINITY;
            }
        }
        float pr[QG][U];
#pragma unroll
        for (int i = 0; i < QG; i++) {
            float m_new = m_run[i];
#pragma unroll
            for (int u = 0; u < U; u++) m_new = fmaxf(m_new, sc[i][u]);
            const float m_safe = m_new == -INFINITY ? 0.f : m_new;  // keeps exp2(-inf - -inf) out of the arithmetic
            const float alpha = __builtin_amdgcn_exp2f(m_run[i] - m_safe);
            float sum = 0.f;
#pragma unroll
            for (int u = 0; u < U; u++) sum += pr[i][u] = __builtin_amdgcn_exp2f(sc[i][u] - m_safe);
            l_run[i] = fmaf(l_run[i], alpha, sum);
            m_run[i] = m_new;
#pragma unroll
            for (int j = 0; j < 8; j++) o[i][j] *= alpha;
        }
#pragma unroll
        for (int u = 0; u < U; u++) {
            float vf[8];
            rows[u].get(vf);
#pragma unroll
            for (int i = 0; i < QG; i++)
#pragma unroll
                for (int j = 0; j < 8; j++) o[i][j] = fmaf(pr[i][u], vf[j], o[i][j]);
        }
    };
    for (int base = t_begin; base < t_end; base += NS * U) {
        fetch(nxt, cs_nxt, base + NS * U);
        absorb(cur, cs_cur, base);
#pragma unroll
        for (int u = 0; u < U; u++) cur[u] = nxt[u], cs_cur[u] = cs_nxt[u];
    }

    // the G streams of the wavefront (lanes with the same c hold the same elements), then the wavefronts through LDS
#pragma unroll
    for (int i = 0; i < QG; i++) {
        const auto add = [](float a, float b) { return a + b; };
        const float mw = over_groups<LPT>(m_run[i], [](float a, float b) { return fmaxf(a, b); });
        const float w = __builtin_amdgcn_exp2f(m_run[i] - (mw == -INFINITY ? 0.f : mw));  // (an empty stream: exp2(-inf) = 0)
        const float lw = over_groups<LPT>(l_run[i] * w, add);
#pragma unroll
        for (int j = 0; j < 8; j++) o[i][j] = over_groups<LPT>(o[i][j] * w, add);
        if (g == 0) {
#pragma unroll
            for (int j = 0; j < 8; j++) so[wave][i][c * 8 + j] = o[i][j];
            if (c == 0) sm[wave][i] = mw, sl[wave][i] = lw;
        }
    }
    __syncthreads();
    for (int e = tid; e < QG * D; e += kThreads) {
        const int i = e / D, d = e - i * D, h = h0 + i;
        if (h >= h_end) continue;
        float m = -INFINITY, acc = 0.f, l = 0.f;
#pragma unroll
        for (int w = 0; w < kWaves; w++) m = fmaxf(m, sm[w][i]);
        const float m_safe = m == -INFINITY ? 0.f : m;
#pragma unroll
        for (int w = 0; w < kWaves; w++) {
            const float f = __builtin_amdgcn_exp2f(sm[w][i] - m_safe);
            acc = fmaf(f, so[w][i][d], acc);
            l = fmaf(f, sl[w][i], l);
        }
        if (p.n_splits > 1) {
            p.opart[((int64_t)split * p.n_head + h) * D + d] = acc;
            if (d == 0) p.ml[2 * (split * p.n_head + h)] = m, p.ml[2 * (split * p.n_head + h) + 1] = l;
        } else if (d < p.dim) {
            const float v = acc / l;
            const int64_t at = (int64_t)row * p.ldo + h * p.dim + d;
            if (p.out_type == SKN_TYPE_F32) ((float*)p.out)[at] = v;
            else ((uint16_t*)p.out)[at] = skn_bf16_bits(v);
        }
    }
}

// one workgroup per row: norms, temperature, the query in its padded layout with the key's norm weights, the key to the cache
template <typename E>
__global__ __launch_bounds__(256) void shared_prep_kernel(const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk,
                                                          const float* __restrict__ q_norm, const float* __restrict__ k_norm, E* __restrict__ pool,
                                                          float* __restrict__ key_scale, const int32_t* __restrict__ table, int page_tokens,
                                                          int n_head, int kv_heads, int dim, int dim_pad, int pos0, float eps, float temp_coef,
                                                          float temp_every, float* __restrict__ q_prep) {
    __shared__ float red[8];
    const int row = blockIdx.x, pos = pos0 + row;
    const float* qr = q + (int64_t)row * ldq;
    const float* kr = k + (int64_t)row * ldk;
    float sq = sum_squares(first_quad(qr, n_head * dim), qr, n_head * dim), sk = sum_squares(first_quad(kr, kv_heads * dim), kr, kv_heads * dim);
    block_sum2(sq, sk, red);
    const float rk = 1.0f / sqrtf(sk / (float)(kv_heads * dim) + eps);
    const float rq = query_temperature(pos, temp_coef, temp_every) / sqrtf(sq / (float)(n_head * dim) + eps);
    const int page = table[pos / page_tokens], slot = pos % page_tokens, per_kv = n_head / kv_heads;
    if (threadIdx.x == 0) key_scale[(int64_t)page * page_tokens + slot] = rk;
    for (int e = threadIdx.x; e < n_head * dim_pad; e += 256) {
        const int h = e / dim_pad, d = e - h * dim_pad;
        q_prep[(int64_t)row * n_head * dim_pad + e] =
            d < dim ? qr[h * dim + d] * rq * q_norm[h * dim + d] * k_norm[h / per_kv * dim + d] : 0.f;
    }
    for (int e = threadIdx.x; e < kv_heads * dim; e += 256) {
        const int h = e / dim, d = e - h * dim;
        const int64_t at = (((int64_t)page * kv_heads + h) * page_tokens + slot) * dim_pad + d;
        if constexpr (sizeof(E) == 4) pool[at] = kr[e];
        else pool[at] = __half_as_ushort(__float2half_rn(kr[e]));
    }
}

// query heads a workgroup of a step takes: as few as keep the workgroups within two per compute unit
int heads_per_group(const skn_ctx* ctx, int per_kv, int kv_heads, int splits) {
    int qg = 1;
    while (qg < 2 && qg * 2 <= per_kv && splits * kv_heads * ((per_kv + qg - 1) / qg) > 2 * ctx->compute_units) qg *= 2;
    return qg;
}

template <typename E, int D, int QG, bool STEP>
int launch_as(skn_ctx* ctx, const AttnArgs& a, int rows) {
    const int per_kv = a.n_head / a.kv_heads;
    skn_launch(ctx, shared_attn_kernel<E, D, QG, STEP>, dim3(a.n_splits, a.kv_heads * ((per_kv + QG - 1) / QG), rows), dim3(kThreads), 0, a);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <int D, bool STEP>
int launch_dim(skn_ctx* ctx, const skn_kv* kv, const AttnArgs& a, int rows) {
    if (kv->elem_type == SKN_TYPE_F32) return launch_as<float, D, 1, STEP>(ctx, a, rows);
    if constexpr (STEP) {
        const int qg = heads_per_group(ctx, a.n_head / a.kv_heads, a.kv_heads, a.n_splits);
        if (qg == 2) return launch_as<uint16_t, D, 2, true>(ctx, a, rows);
    }
    return launch_as<uint16_t, D, 1, STEP>(ctx, a, rows);
}

template <bool STEP>
int launch_attn(skn_ctx* ctx, const skn_kv* kv, const AttnArgs& a, int rows) {
    if (kv->head_dim == 64) return launch_dim<64, STEP>(ctx, kv, a, rows);
    if (kv->head_dim == 128) return launch_dim<128, STEP>(ctx, kv, a, rows);
    return launch_dim<256, STEP>(ctx, kv, a, rows);
}

AttnArgs base_args(const skn_kv* kv, int seq, const skn_shared_attn& p) {
    AttnArgs a = {};
    a.pool = kv->k_pool;
    a.key_scale = kv->key_scale;
    a.table = kv->page_table_dev + (size_t)seq * kv->pages_per_seq;
    a.page_tokens = kv->page_tokens;
    a.pages_per_seq = kv->pages_per_seq;
    a.inv_page = 1.0f / (float)kv->page_tokens;
    a.n_head = p.n_head;
    a.kv_heads = kv->n_head;
    a.dim = kv->dim;
    a.scale_log2e = p.scale * kLog2e;
    a.n_splits = 1;
    a.q_norm = p.q_norm;
    a.k_norm = p.k_norm;
    a.eps = p.eps;
    a.temp_coef = p.temp_coef;
    a.temp_every = p.temp_every;
    return a;
}

int check(skn_ctx* ctx, const skn_kv* kv, const skn_shared_attn& p) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_SHARED, SKN_ERR_STATE, "shared attention: the cache keeps keys and values apart");
    SKN_REQUIRE(ctx, p.n_head > 0 && p.n_head % kv->n_head == 0, SKN_ERR_SHAPE, "shared attention: %d query heads over %d cached heads", p.n_head, kv->n_head);
    SKN_REQUIRE(ctx, p.q_norm && p.k_norm && (p.temp_coef == 0.f || p.temp_every > 0.f), SKN_ERR_ARG, "shared attention: bad parameters");
    return SKN_OK;
}

}  // namespace

int skn_shared_prep_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q, int ldq, const float* k, int ldk, int n,
                         int pos0, float* q_prep) {
    SKN_TRY(check(ctx, kv, p));
    const int32_t* table = kv->page_table_dev + (size_t)seq * kv->pages_per_seq;
    if (kv->elem_type == SKN_TYPE_F32)
        skn_launch(ctx, shared_prep_kernel<float>, dim3(n), dim3(256), 0, q, ldq, k, ldk, p.q_norm, p.k_norm, (float*)kv->k_pool, kv->key_scale, table,
                   kv->page_tokens, p.n_head, kv->n_head, kv->dim, kv->head_dim, pos0, p.eps, p.temp_coef, p.temp_every, q_prep);
    else
        skn_launch(ctx, shared_prep_kernel<uint16_t>, dim3(n), dim3(256), 0, q, ldq, k, ldk, p.q_norm, p.k_norm, kv->k_pool, kv->key_scale, table,
                   kv->page_tokens, p.n_head, kv->n_head, kv->dim, kv->head_dim, pos0, p.eps, p.temp_coef, p.temp_every, q_prep);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_shared_attn_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q_prep, int n, int pos0, void* out, int ldo,
                         int out_type) {
    SKN_TRY(check(ctx, kv, p));
    if (kv->elem_type == SKN_TYPE_F16 && kv->head_dim <= 128)
        return skn_shared_attn_prefill_launch(ctx, kv, seq, q_prep, n, pos0 + 1, p.n_head, p.scale, out, ldo, out_type);
    AttnArgs a = base_args(kv, seq, p);
    a.out = out;
    a.ldo = ldo;
    a.out_type = out_type;
    for (int z = 0; z < n; z += 32768) {  // (grid limit)
        a.q_prep = q_prep + (int64_t)z * p.n_head * kv->head_dim;
        a.first_ctx = pos0 + z + 1;
        a.out = (uint8_t*)out + (int64_t)z * ldo * (out_type == SKN_TYPE_F32 ? 4 : 2);
        SKN_TRY(launch_attn<false>(ctx, kv, a, std::min(n - z, 32768)));
    }
    return SKN_OK;
}

int skn_shared_attn_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q, const float* k, const int32_t* state_dev,
                         int n_splits, float* opart, float* ml, float* out) {
    SKN_TRY(check(ctx, kv, p));
    SKN_REQUIRE(ctx, n_splits >= 1 && n_splits <= kMaxSplits && (n_splits == 1 ? out != nullptr : opart && ml), SKN_ERR_ARG,
                "shared attention: %d splits without their buffers", n_splits);
    AttnArgs a = base_args(kv, seq, p);
    a.q = q;
    a.k = k;
    a.state = state_dev;
    a.n_splits = n_splits;
    a.opart = opart;
    a.ml = ml;
    a.out = out;
    a.out_type = SKN_TYPE_F32;
    return launch_attn<true>(ctx, kv, a, 1);
}

// Splits for contexts up to max_ctx: a power of two, at most eight (sixteen where few heads would read a long context: the
// merge reads every split in every workgroup that follows), so that a workgroup has at least a round of requests.
int skn_shared_attn_splits(skn_ctx* ctx, const skn_kv* kv, int n_head, int max_ctx) {
    const int round = kWaves * 512 / kv->head_dim * kU;
    const int most = n_head * 8 <= ctx->compute_units / 2 ? kMaxSplits : 8;
    int n = 1;
    while (n < most && n * round < max_ctx) n *= 2;
    return n;
}

extern "C" int skn_attn_shared(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn* p, const float* q_dev, const float* k_dev, int n,
                               float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_attn_shared: ctx is null");
    SKN_REQUIRE(ctx, kv && p && q_dev && k_dev && out_dev, SKN_ERR_ARG, "skn_attn_shared: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < kv->n_seq && n > 0, SKN_ERR_RANGE, "skn_attn_shared: %d tokens of sequence %d of %d", n, seq, kv->n_seq);
    SKN_TRY(check(ctx, kv, *p));
    const int pos0 = kv->len[seq];
    SKN_TRY(skn_kv_reserve(ctx, kv, seq, pos0 + n));
    float* q_prep = nullptr;
    SKN_HIP(ctx, hipMalloc((void**)&q_prep, (size_t)n * p->n_head * kv->head_dim * sizeof(float)));
    int rc = skn_shared_prep_rows(ctx, kv, seq, *p, q_dev, p->n_head * kv->dim, k_dev, kv->n_head * kv->dim, n, pos0, q_prep);
    if (rc == SKN_OK) rc = skn_shared_attn_rows(ctx, kv, seq, *p, q_prep, n, pos0, out_dev, p->n_head * kv->dim, SKN_TYPE_F32);
    if (rc == SKN_OK) rc = skn_kv_advance_len(ctx, kv, seq, n);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(q_prep);
    return rc;
}
