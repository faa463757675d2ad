// Latent attention: one cached row per token for all heads -- the normed latent c and a rotated key part.
//
//   score = scale (q . Wuk c + q_rot . k_rot),   out = Wuv sum softmax(score) c
//
// A decode step (and a prompt over an fp32 cache) never expands a key: Wuk^T q takes the query to the latent's space, where the
// cached row is key and, in its first part, value; Wuv follows the weighted sum.  Three launches: [queries to the latent's space,
// their rotation, the token's own row to the cache], the rows streamed once per head (attention_stream.h), [merge of the splits,
// values].  A prompt expands keys and values of the tokens that its queries see with one GEMM and goes through the matrix cores
// (csrc/attention_prefill.hip), which takes a third of the operations per key.
#include "attention_stream.h"

#include <algorithm>

namespace {

constexpr int kMaxSplits = 16;

template <typename W>
__device__ __forceinline__ void load_weights8(const W* p, float (&f)[8]) {
    if constexpr (sizeof(W) == 4) {
        const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
        f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w, f[4] = b.x, f[5] = b.y, f[6] = b.z, f[7] = b.w;
    } else {
        const u32x4 a = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
        for (int j = 0; j < 4; j++) f[2 * j] = __uint_as_float(a[j] << 16), f[2 * j + 1] = __uint_as_float(a[j] & 0xFFFF0000u);
    }
}

struct LatentArgs {
    skn_latent_attn p;
    int rank_pad, width;  // columns of w_up; elements of a cached row and of a prepared query
    const float* q;
    int ldq;
    const float* d;
    int ldd;
    void* pool;
    const int32_t* table;
    int page_tokens, pos0;
    const int32_t* state;  // a step's position at [1], or null: row z is at pos0 + z
    float* q_prep;
};

// the token's own row: latent divided by its root mean square, the key part rotated; the whole workgroup
template <typename E>
__device__ __forceinline__ void store_latent_row(const LatentArgs& a, int row, int pos, float* red) {
    const int tid = threadIdx.x, nt = blockDim.x, rank = a.p.rank, half = a.p.rot_dim >> 1;
    const float* d = a.d + (int64_t)row * a.ldd;
    float ss = 0.f;
    for (int i = tid; i < rank; i += nt) ss = fmaf(d[i], d[i], ss);
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    ss = 0.f;
    for (int i = 0; i < nt >> 6; i++) ss += red[i];
    const float f = 1.0f / sqrtf(ss / (float)rank + a.p.eps);
    E* dst = (E*)a.pool + ((int64_t)a.table[pos / a.page_tokens] * a.page_tokens + pos % a.page_tokens) * a.width;
    for (int i = tid; i < rank; i += nt) store_cached(dst + i, d[i] * f * a.p.norm[i]);
    for (int i = tid; i < half; i += nt) {
        float sn, cs;
        skn_rope_sincos_freq(pos, a.p.rot_freq[i], &sn, &cs);
        const float u = d[rank + i], v = d[rank + half + i];
        store_cached(dst + rank + i, u * cs - v * sn);
        store_cached(dst + rank + half + i, v * cs + u * sn);
    }
}

// grid (heads (+ 1: the row to the cache), rows), sixteen wavefronts: wavefront w takes every sixteenth row of Wuk, a lane eight of its
// columns.  LDS: [16][rank_pad].
template <typename E, typename W>
__global__ __launch_bounds__(1024) void latent_prep_kernel(const LatentArgs a) {
    extern __shared__ __align__(16) float part[];
    __shared__ float qs[256], red[16];
    const int h = blockIdx.x, row = blockIdx.y, pos = a.state ? a.state[1] : a.pos0 + row, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    if (h == a.p.n_head) {
        store_latent_row<E>(a, row, pos, red);
        return;
    }
    const int dim = a.p.dim, rank = a.p.rank, half = a.p.rot_dim >> 1, pieces = a.rank_pad >> 3;
    const float* q = a.q + (int64_t)row * a.ldq + h * (dim + a.p.rot_dim);
    float* out = a.q_prep + ((int64_t)row * a.p.n_head + h) * a.width;
    if (tid < dim) qs[tid] = q[tid];
    for (int i = tid; i < half; i += 1024) {
        float sn, cs;
        skn_rope_sincos_freq(pos, a.p.rot_freq[i], &sn, &cs);
        const float u = q[dim + i], v = q[dim + half + i];
        out[rank + i] = u * cs - v * sn;
        out[rank + half + i] = v * cs + u * sn;
    }
    for (int i = rank + a.p.rot_dim + tid; i < a.width; i += 1024) out[i] = 0.f;
    __syncthreads();
    const W* w = (const W*)a.p.w_up + (int64_t)h * dim * a.rank_pad;
    for (int pc = lane; pc < pieces; pc += 64) {
        float acc[8];
#pragma unroll
        for (int e = 0; e < 8; e++) acc[e] = 0.f;
#pragma unroll 4
        for (int i = wave; i < dim; i += 16) {
            float f[8];
            load_weights8(w + (int64_t)i * a.rank_pad + 8 * pc, f);
            const float x = qs[i];
#pragma unroll
            for (int e = 0; e < 8; e++) acc[e] = fmaf(x, f[e], acc[e]);
        }
        float4* dst = reinterpret_cast<float4*>(part + wave * a.rank_pad + 8 * pc);
        dst[0] = make_float4(acc[0], acc[1], acc[2], acc[3]);
        dst[1] = make_float4(acc[4], acc[5], acc[6], acc[7]);
    }
    __syncthreads();
    for (int i = tid; i < rank; i += 1024) {
        float s = 0.f;
#pragma unroll
        for (int k = 0; k < 16; k++) s += part[k * a.rank_pad + i];
        out[i] = s;
    }
}

constexpr int kValueRows = 32;
// grid (heads, rows, rows of Wuv / 32), eight wavefronts: the head's latent (merged from the splits) in LDS, then four rows of Wuv per
// wavefront
template <typename W>
__global__ __launch_bounds__(512) void latent_value_kernel(const skn_latent_attn p, int row0, int rank_pad, int width, const float* __restrict__ lat, int splits,
                                                           const float* __restrict__ ml, void* __restrict__ out, int ldo, int out_type) {
    extern __shared__ __align__(16) float x[];  // [rank_pad]
    const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, rank = p.rank;
    if (splits > 1) {
        float m = -INFINITY, l = 0.f, f[kMaxSplits];
        float2 part[kMaxSplits];  // (all requested before the first is used)
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) part[i] = reinterpret_cast<const float2*>(ml)[min(i, splits - 1) * p.n_head + h];
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) m = fmaxf(m, part[i].x);
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) {
            f[i] = i < splits ? __builtin_amdgcn_exp2f(part[i].x - m) : 0.f;
            l = fmaf(f[i], part[i].y, l);
        }
        const float inv = 1.0f / l;
        for (int i = tid; i < rank_pad; i += 512) {
            float a = 0.f;
            if (i < rank) {
                float y[kMaxSplits];
#pragma unroll
                for (int s = 0; s < kMaxSplits; s++) y[s] = lat[((int64_t)min(s, splits - 1) * p.n_head + h) * width + i];
#pragma unroll
                for (int s = 0; s < kMaxSplits; s++) a = fmaf(f[s], y[s], a);
            }
            x[i] = a * inv;
        }
    } else {
        for (int i = tid; i < rank_pad; i += 512) x[i] = i < rank ? lat[((int64_t)row * p.n_head + h) * rank + i] : 0.f;
    }
    __syncthreads();
    const W* w = (const W*)p.w_up + ((int64_t)row0 + h * p.vdim) * rank_pad;
    const int v0 = blockIdx.z * kValueRows + wave * 4;
    float s[4] = {0.f, 0.f, 0.f, 0.f};
    for (int pc = lane; pc < rank_pad >> 3; pc += 64) {
        float f[4][8];
#pragma unroll
        for (int r = 0; r < 4; r++) load_weights8(w + (int64_t)min(v0 + r, p.vdim - 1) * rank_pad + 8 * pc, f[r]);
        const float4 a = reinterpret_cast<const float4*>(x)[2 * pc], b = reinterpret_cast<const float4*>(x)[2 * pc + 1];
#pragma unroll
        for (int r = 0; r < 4; r++)
            s[r] += ((f[r][0] * a.x + f[r][1] * a.y) + (f[r][2] * a.z + f[r][3] * a.w)) + ((f[r][4] * b.x + f[r][5] * b.y) + (f[r][6] * b.z + f[r][7] * b.w));
    }
#pragma unroll
    for (int r = 0; r < 4; r++) {
        s[r] = wave_sum(s[r]);
        if (lane != 0 || v0 + r >= p.vdim) continue;
        const int64_t at = (int64_t)row * ldo + h * p.vdim + v0 + r;
        if (out_type == SKN_TYPE_F32) ((float*)out)[at] = s[r];
        else ((uint16_t*)out)[at] = skn_bf16_bits(s[r]);
    }
}

// ---- prompts through expanded keys ------------------------------------------------------------------------------------------

// one workgroup per row: the row to the cache (with d), queries rotated into rows of kwidth
__global__ __launch_bounds__(256) void latent_query_kernel(const LatentArgs a, int kwidth) {
    __shared__ float red[16], sn[128], cs[128];
    const int row = blockIdx.x, pos = a.pos0 + row, tid = threadIdx.x, dim = a.p.dim, half = a.p.rot_dim >> 1, qd = dim + a.p.rot_dim;
    if (tid < half) skn_rope_sincos_freq(pos, a.p.rot_freq[tid], &sn[tid], &cs[tid]);
    if (a.d) store_latent_row<uint16_t>(a, row, pos, red);
    __syncthreads();
    const float* q = a.q + (int64_t)row * a.ldq;
    for (int e = tid; e < a.p.n_head * kwidth; e += 256) {
        const int h = e / kwidth, i = e - h * kwidth;
        const float* x = q + h * qd;
        float y = 0.f;
        if (i < dim) y = x[i];
        else if (i < dim + half) y = x[i] * cs[i - dim] - x[i + half] * sn[i - dim];
        else if (i < qd) y = x[i] * cs[i - dim - half] + x[i - half] * sn[i - dim - half];
        a.q_prep[(int64_t)row * a.p.n_head * kwidth + e] = y;
    }
}

// cached rows of the tokens token0 .. : latents as bf16 rows of rank_pad for the GEMM, rotated parts as they are
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ pool, const int32_t* __restrict__ table, int page_tokens, int width,
                                                            int rank, int rank_pad, int rot_dim, int token0, uint16_t* __restrict__ c,
                                                            uint16_t* __restrict__ rot) {
    const int i = blockIdx.x, t = token0 + i;
    const uint16_t* src = pool + ((int64_t)table[t / page_tokens] * page_tokens + t % page_tokens) * width;
    for (int e = threadIdx.x; e < rank_pad; e += 256) c[(int64_t)i * rank_pad + e] = e < rank ? skn_bf16_bits(h2f_bits(src[e])) : 0;
    for (int e = threadIdx.x; e < rot_dim; e += 256) rot[(int64_t)i * rot_dim + e] = src[rank + e];
}

int check(skn_ctx* ctx, const skn_kv* kv, const skn_latent_attn& p, bool own) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_LATENT, SKN_ERR_STATE, "latent attention: not a latent cache");
    SKN_REQUIRE(ctx, p.n_head > 0 && p.dim > 0 && p.dim <= 256 && p.vdim > 0 && p.vdim <= 256, SKN_ERR_SHAPE, "latent attention: %d heads of %d and %d elements",
                p.n_head, p.dim, p.vdim);
    SKN_REQUIRE(ctx, p.rank == kv->vdim && p.rank + p.rot_dim == kv->dim, SKN_ERR_SHAPE, "latent attention: rows of %d + %d elements in a cache of %d + %d", p.rank,
                p.rot_dim, kv->vdim, kv->dim - kv->vdim);
    SKN_REQUIRE(ctx, p.w_up && (!own || p.norm) && (p.rot_dim == 0 || p.rot_freq) && ((uintptr_t)p.w_up & 15) == 0, SKN_ERR_ARG, "latent attention: missing weights");
    SKN_REQUIRE(ctx, p.w_type == SKN_TYPE_BF16 || p.w_type == SKN_TYPE_F32, SKN_ERR_TYPE, "latent attention: weights of type %d (BF16 or F32)", p.w_type);
    SKN_REQUIRE(ctx, p.mask == SKN_MASK_CAUSAL || ((p.mask == SKN_MASK_WINDOW || p.mask == SKN_MASK_CHUNK) && p.mask_size > 0), SKN_ERR_ARG,
                "latent attention: mask %d of %d tokens", p.mask, p.mask_size);
    return SKN_OK;
}

LatentArgs latent_args(const skn_kv* kv, int seq, const skn_latent_attn& p, const float* q, int ldq, const float* d, int ldd) {
    LatentArgs a = {};
    a.p = p;
    a.rank_pad = skn_pad_cols(p.rank);
    a.width = kv->head_dim;
    a.q = q;
    a.ldq = ldq;
    a.d = d;
    a.ldd = ldd;
    a.pool = kv->k_pool;
    a.table = kv->page_table_dev + (size_t)seq * kv->pages_per_seq;
    a.page_tokens = kv->page_tokens;
    return a;
}

template <typename E, typename W>
int launch_prep(skn_ctx* ctx, const LatentArgs& a, int rows) {
    skn_launch(ctx, latent_prep_kernel<E, W>, dim3(a.p.n_head + (a.d ? 1 : 0), rows), dim3(1024), (size_t)16 * a.rank_pad * sizeof(float), a);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int prep(skn_ctx* ctx, const skn_kv* kv, const LatentArgs& a, int rows) {
    const bool bf16 = a.p.w_type == SKN_TYPE_BF16;
    if (kv->elem_type == SKN_TYPE_F32) return bf16 ? launch_prep<float, uint16_t>(ctx, a, rows) : launch_prep<float, float>(ctx, a, rows);
    return bf16 ? launch_prep<uint16_t, uint16_t>(ctx, a, rows) : launch_prep<uint16_t, float>(ctx, a, rows);
}

StreamArgs latent_stream(const skn_kv* kv, int seq, const skn_latent_attn& p, const float* q_prep) {
    StreamArgs a = stream_args(kv, seq, p.n_head);
    a.kv_heads = 1;
    a.scale = p.scale;
    a.range.kind = p.mask;
    a.range.size = p.mask_size;
    a.q_prep = q_prep;
    return a;
}

template <typename E>
int launch_stream(skn_ctx* ctx, const skn_kv* kv, const StreamArgs& a, int rows) {
    const dim3 grid(a.n_splits, a.n_head, rows), block(stream_threads<kStreamLatent>());
    switch (kv->head_dim / 128) {
        case 1: skn_launch(ctx, stream_attn_kernel<E, 16, 1, kStreamLatent>, grid, block, 0, a); break;
        case 2: skn_launch(ctx, stream_attn_kernel<E, 16, 2, kStreamLatent>, grid, block, 0, a); break;
        case 3: skn_launch(ctx, stream_attn_kernel<E, 16, 3, kStreamLatent>, grid, block, 0, a); break;
        case 5: skn_launch(ctx, stream_attn_kernel<E, 16, 5, kStreamLatent>, grid, block, 0, a); break;
        default: skn_launch(ctx, stream_attn_kernel<E, 16, 8, kStreamLatent>, grid, block, 0, a); break;
    }
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int stream(skn_ctx* ctx, const skn_kv* kv, const StreamArgs& a, int rows) {
    return kv->elem_type == SKN_TYPE_F32 ? launch_stream<float>(ctx, kv, a, rows) : launch_stream<uint16_t>(ctx, kv, a, rows);
}

int value(skn_ctx* ctx, const skn_kv* kv, const skn_latent_attn& p, const float* lat, int splits, const float* ml, int rows, void* out, int ldo, int out_type) {
    const int rank_pad = skn_pad_cols(p.rank), row0 = skn_pad_rows(p.n_head * p.dim);  // (of Wuv)
    const dim3 grid(p.n_head, rows, (p.vdim + kValueRows - 1) / kValueRows);
    const size_t lds = (size_t)rank_pad * sizeof(float);
    if (p.w_type == SKN_TYPE_F32) skn_launch(ctx, latent_value_kernel<float>, grid, dim3(512), lds, p, row0, rank_pad, kv->head_dim, lat, splits, ml, out, ldo, out_type);
    else skn_launch(ctx, latent_value_kernel<uint16_t>, grid, dim3(512), lds, p, row0, rank_pad, kv->head_dim, lat, splits, ml, out, ldo, out_type);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

// the padded key width of the matrix-core form, or 0
int expanded_width(const skn_kv* kv, const skn_latent_attn& p) {
    return kv->elem_type == SKN_TYPE_F16 && p.w_type == SKN_TYPE_BF16 ? skn_latent_prefill_width(p.dim, p.rot_dim, p.vdim) : 0;
}

int expanded_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn& p, LatentArgs& a, int kwidth, int n, skn_latent_ws* ws, void* out, int ldo,
                  int out_type) {
    skn_launch(ctx, latent_query_kernel, dim3(n), dim3(256), 0, a, kwidth);
    SKN_LAUNCH_CHECK(ctx);
    skn_prefill_ranged r;
    r.range.kind = p.mask;
    r.range.size = p.mask_size;
    const int token0 = r.range.first(a.pos0) & ~31, tokens = a.pos0 + n - token0;
    const int kcols = skn_pad_rows(p.n_head * p.dim), vcols = skn_pad_rows(p.n_head * p.vdim);
    auto up = [](size_t b) { return (b + 255) & ~(size_t)255; };
    const size_t cb = up((size_t)tokens * a.rank_pad * 2), rb = up((size_t)tokens * p.rot_dim * 2), kb = up((size_t)tokens * kcols * 2),
                 vb = up((size_t)tokens * vcols * 2), need = cb + rb + kb + vb;
    if (need > ws->bytes) {
        SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
        if (ws->mem) SKN_HIP(ctx, hipFree(ws->mem));
        ws->mem = nullptr;
        ws->bytes = 0;
        hipError_t e = hipMalloc(&ws->mem, need);
        if (e != hipSuccess) {
            (void)hipGetLastError();
            return skn_fail(ctx, SKN_ERR_OOM, "latent attention: %zu bytes of workspace: %s", need, hipGetErrorString(e));
        }
        ws->bytes = need;
    }
    uint8_t* at = (uint8_t*)ws->mem;
    uint16_t *c = (uint16_t*)at, *rot = (uint16_t*)(at + cb), *k = (uint16_t*)(at + cb + rb), *v = (uint16_t*)(at + cb + rb + kb);
    skn_launch(ctx, latent_gather_kernel, dim3(tokens), dim3(256), 0, (const uint16_t*)kv->k_pool, a.table, kv->page_tokens, kv->head_dim, p.rank, a.rank_pad,
               p.rot_dim, token0, c, rot);
    SKN_LAUNCH_CHECK(ctx);
    skn_dense_mat w;
    w.w = p.w_up;
    w.type = p.w_type;
    w.rows = kcols + vcols;
    w.k_pad = a.rank_pad;
    skn_dense_out o;
    o.seg[o.nseg++] = {0, p.n_head * p.dim, SKN_OP_NONE, 0.f, 0.f, k, kcols, SKN_TYPE_F16};
    o.seg[o.nseg++] = {kcols, p.n_head * p.vdim, SKN_OP_NONE, 0.f, 0.f, v, vcols, SKN_TYPE_F16};
    SKN_TRY(skn_dense_gemm(ctx, w, c, a.rank_pad, tokens, o));
    r.scale = p.scale;
    r.vdim = p.vdim;
    r.out = out;
    r.ldo = ldo;
    r.out_type = out_type;
    return skn_latent_prefill_launch(ctx, k, kcols, rot, v, vcols, p.dim, p.rot_dim, token0, a.q_prep, n, a.pos0, p.n_head, r);
}

int latent_init(skn_ctx* ctx) {  // (16 x 1024 floats and more than the default of 64 KiB)
    const void* f[4] = {(const void*)latent_prep_kernel<float, float>, (const void*)latent_prep_kernel<float, uint16_t>,
                        (const void*)latent_prep_kernel<uint16_t, float>, (const void*)latent_prep_kernel<uint16_t, uint16_t>};
    for (const void* k : f) SKN_HIP(ctx, hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, 16 * 1024 * 4));
    return SKN_OK;
}
skn_family register_family(latent_init);

}  // namespace

size_t skn_latent_prep_floats(const skn_kv* kv, const skn_latent_attn& p) { return (size_t)p.n_head * std::max(kv->head_dim, expanded_width(kv, p)); }
size_t skn_latent_lat_floats(const skn_kv* kv, const skn_latent_attn& p) { return expanded_width(kv, p) ? 0 : (size_t)p.n_head * p.rank; }

int skn_latent_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn& p, const float* q, int ldq, const float* d, int ldd, int n, int pos0,
                    float* q_prep, float* lat, skn_latent_ws* ws, void* out, int ldo, int out_type) {
    SKN_TRY(check(ctx, kv, p, d != nullptr));
    LatentArgs a = latent_args(kv, seq, p, q, ldq, d, ldd);
    a.q_prep = q_prep;
    a.pos0 = pos0;
    const int kwidth = expanded_width(kv, p);
    if (kwidth) return expanded_rows(ctx, kv, seq, p, a, kwidth, n, ws, out, ldo, out_type);
    // (the cache rows of all n tokens are written before the first of them is read: the launches follow each other)
    for (int z = 0; z < n; z += 32768) {  // (grid limit)
        const int rows = std::min(n - z, 32768);
        LatentArgs b = a;
        b.q = q + (int64_t)z * ldq;
        b.d = d ? d + (int64_t)z * ldd : nullptr;
        b.pos0 = pos0 + z;
        b.q_prep = q_prep + (int64_t)z * p.n_head * kv->head_dim;
        SKN_TRY(prep(ctx, kv, b, rows));
        StreamArgs s = latent_stream(kv, seq, p, b.q_prep);
        s.first_ctx = pos0 + z + 1;
        s.out = lat + (int64_t)z * p.n_head * p.rank;
        s.ldo = p.n_head * p.rank;
        s.out_type = SKN_TYPE_F32;
        SKN_TRY(stream(ctx, kv, s, rows));
        SKN_TRY(value(ctx, kv, p, (const float*)s.out, 1, nullptr, rows, (uint8_t*)out + (int64_t)z * ldo * (out_type == SKN_TYPE_F32 ? 4 : 2), ldo, out_type));
    }
    return SKN_OK;
}

int skn_latent_splits(skn_ctx* ctx, const skn_kv* kv, const skn_latent_attn& p, int max_ctx) {
    skn_range r;
    r.kind = p.mask;
    r.size = p.mask_size;
    const int streams = 8 * 4 * (kv->elem_type == SKN_TYPE_F32 || kv->head_dim > 640 ? 1 : 2);  // (rows of a workgroup and round)
    return skn_ranged_splits(ctx, p.n_head, 2 * streams, r, max_ctx);
}

int skn_latent_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn& p, const float* q, const float* d, const int32_t* state_dev, int n_splits,
                    float* q_prep, float* opart, float* ml, float* out) {
    SKN_TRY(check(ctx, kv, p, d != nullptr));
    SKN_REQUIRE(ctx, n_splits >= 1 && n_splits <= kMaxSplits && q_prep && opart && ml && out, SKN_ERR_ARG, "latent attention: %d splits without their buffers", n_splits);
    LatentArgs a = latent_args(kv, seq, p, q, 0, d, 0);
    a.q_prep = q_prep;
    a.state = state_dev;
    SKN_TRY(prep(ctx, kv, a, 1));
    StreamArgs s = latent_stream(kv, seq, p, q_prep);
    s.state = state_dev;
    s.n_splits = n_splits;
    s.opart = opart;
    s.ml = ml;
    s.out = opart;
    s.ldo = p.n_head * p.rank;
    s.out_type = SKN_TYPE_F32;
    SKN_TRY(stream(ctx, kv, s, 1));
    return value(ctx, kv, p, opart, n_splits, ml, 1, out, 0, SKN_TYPE_F32);
}

extern "C" int skn_attn_latent(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn* p, const float* q_dev, const float* d_dev, int n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_attn_latent: ctx is null");
    SKN_REQUIRE(ctx, kv && p && q_dev && out_dev, SKN_ERR_ARG, "skn_attn_latent: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < kv->n_seq && n > 0, SKN_ERR_RANGE, "skn_attn_latent: %d tokens of sequence %d of %d", n, seq, kv->n_seq);
    SKN_REQUIRE(ctx, d_dev || n <= kv->len[seq], SKN_ERR_RANGE, "skn_attn_latent: %d tokens again of %d", n, kv->len[seq]);
    SKN_TRY(check(ctx, kv, *p, d_dev != nullptr));
    const int pos0 = d_dev ? kv->len[seq] : kv->len[seq] - n;
    SKN_TRY(skn_kv_reserve(ctx, kv, seq, pos0 + n));
    const size_t prep_floats = (size_t)n * skn_latent_prep_floats(kv, *p), lat_floats = std::max((size_t)n * skn_latent_lat_floats(kv, *p), (size_t)p->n_head * kv->head_dim),
                 ml_floats = 32 * (size_t)p->n_head;
    float* scratch = nullptr;
    SKN_HIP(ctx, hipMalloc((void**)&scratch, (prep_floats + lat_floats + ml_floats + 4) * sizeof(float)));
    float *lat = scratch + prep_floats, *ml = lat + lat_floats;
    skn_latent_ws ws;
    int rc;
    if (n == 1) {
        const int32_t state[4] = {0, pos0, pos0 + 1, 0};
        rc = skn_upload(ctx, ml + ml_floats, state, sizeof(state));
        if (rc == SKN_OK) rc = skn_latent_step(ctx, kv, seq, *p, q_dev, d_dev, (const int32_t*)(ml + ml_floats), 1, scratch, lat, ml, out_dev);
    } else {
        rc = skn_latent_rows(ctx, kv, seq, *p, q_dev, p->n_head * (p->dim + p->rot_dim), d_dev, p->rank + p->rot_dim, n, pos0, scratch, lat, &ws, out_dev,
                             p->n_head * p->vdim, SKN_TYPE_F32);
    }
    if (rc == SKN_OK && d_dev) rc = skn_kv_advance_len(ctx, kv, seq, n);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(scratch);
    if (ws.mem) (void)hipFree(ws.mem);
    return rc;
}
