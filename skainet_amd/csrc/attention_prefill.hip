// Causal attention of many query rows of one sequence (prompt processing) on the matrix cores.
//
//   out[t, h, :] = softmax(q[t, h, :] . K[0 : n_t, h, :]^T * scale) . V[0 : n_t, h, :],   n_t = first_ctx + t
//
// Two launches.  (1) attn_frag_kernel copies the K and V rows of the sequence out of the paged cache into the
// order in which the matrix instructions take them: per head and tile of 32 tokens, the 64 lanes x 16 bytes of
// every operand are contiguous (K as the row operand of K . Q^T, V transposed as the row operand of V^T . P^T),
// so the attention kernel loads an operand with one coalesced 1 KiB load and uses neither LDS nor barriers.
// (2) attn_prefill_kernel: one workgroup of four wavefronts per (32 query rows, head); wavefront w walks the key
// tiles w, w + 4, ... up to the causal limit with the online softmax, and the four partial results are merged
// through LDS: S^T = K Q^T (scores of a query sit in one lane column: its maximum and sum need no
// cross-lane traffic beyond the two lane halves), P = exp2(S - max), O^T += V^T P^T.
// A query may see a range of the keys only (a window, or its chunk): tiles outside the range of a block of queries are neither copied
// nor visited.  Latents come expanded: attn_frag_rows_kernel takes their keys and values row by row.
// Precision: K and V are the cached fp16 values; q (pre-multiplied by scale * log2 e) and P enter as fp16 pairs
// hi + lo (two matrix instructions per step), products and sums are fp32.
#include "kv.h"
#include "dense.h"

namespace {

typedef _Float16 half8_t __attribute__((ext_vector_type(8)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float float16_t __attribute__((ext_vector_type(16)));

// In the accumulator layout of v_mfma_f32_32x32x16_f16, register x of lane l = 32 h + n holds row
// 8 (x / 4) + 4 h + x % 4 of column n.  Registers 0..7 (8..15) of the score tile are handed on as the eight k
// values of lane half h in the first (second) k-step of the next product, so position p of half h in k-step s
// stands for key 16 s + 8 (p / 4) + 4 h + p % 4 of the tile -- the V^T operand is written in that key order.
__device__ __forceinline__ int key_of(int s, int h, int p) { return 16 * s + 8 * (p >> 2) + 4 * h + (p & 3); }

// grid (tiles, heads), 256 threads; tile i holds the tokens from 32 (tile0 + i) on.  Tokens at or beyond n_tokens are written as
// zeros.
// kfrag: [head][tile][k-step D/16][lane] x 8 halves: lane 32 h + r = elements 16 s + 8 h .. + 7 of key r.
// vfrag: [head][tile][32-row block of d][k-step 2][lane] x 8 halves: lane 32 h + r = element 32 b + r of the
//        eight keys key_of(s, h, 0..7).
// SHARED: a cache that shares its keys and values (kv.h): the row is the value, and times its token's key_scale the key.
template <int D, bool SHARED>
__global__ __launch_bounds__(256) void attn_frag_kernel(const uint16_t* __restrict__ k_pool, const uint16_t* __restrict__ v_pool,
                                                        const float* __restrict__ key_scale, const int32_t* __restrict__ table,
                                                        int n_head, int page_tokens,
                                                        int n_tokens, int tile0, int n_tiles, u32x4* __restrict__ kfrag,
                                                        u32x4* __restrict__ vfrag) {
    constexpr int kPieces = D / 8;             // 16-byte pieces of a row
    constexpr int kPitch = D + 8;              // LDS row pitch in halves
    __shared__ __align__(16) uint16_t vt[32 * kPitch];
    const int tile = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    u32x4* kout = kfrag + ((size_t)head * n_tiles + tile) * (D / 16) * 64;
    u32x4* vout = vfrag + ((size_t)head * n_tiles + tile) * (D / 16) * 64;
    for (int i = tid; i < 32 * kPieces; i += 256) {
        const int r = i / kPieces, pc = i - r * kPieces;
        const int t = 32 * (tile0 + tile) + r;
        u32x4 kk = {0u, 0u, 0u, 0u}, vv = kk;
        if (t < n_tokens) {
            const int page = table[t / page_tokens], slot = t % page_tokens;
            const size_t off = (((size_t)page * n_head + head) * page_tokens + slot) * D + 8 * pc;
            kk = *reinterpret_cast<const u32x4*>(k_pool + off);
            if constexpr (SHARED) {
                vv = kk;
                const float f = key_scale[(size_t)page * page_tokens + slot];
                half8_t x = __builtin_bit_cast(half8_t, kk);
#pragma unroll
                for (int e = 0; e < 8; e++) x[e] = (_Float16)((float)x[e] * f);
                kk = __builtin_bit_cast(u32x4, x);
            } else {
                vv = *reinterpret_cast<const u32x4*>(v_pool + off);
            }
        }
        kout[(pc >> 1) * 64 + 32 * (pc & 1) + r] = kk;
        *reinterpret_cast<u32x4*>(vt + r * kPitch + 8 * pc) = vv;
    }
    __syncthreads();
    for (int i = tid; i < (D / 32) * 2 * 64; i += 256) {
        const int lane = i & 63, s = (i >> 6) & 1, b = i >> 7;
        const int h = lane >> 5, r = lane & 31;
        uint32_t w[4];
#pragma unroll
        for (int p = 0; p < 8; p += 2) {
            const uint32_t lo = vt[key_of(s, h, p) * kPitch + 32 * b + r], hi = vt[key_of(s, h, p + 1) * kPitch + 32 * b + r];
            w[p >> 1] = lo | (hi << 16);
        }
        vout[i] = u32x4{w[0], w[1], w[2], w[3]};
    }
}

// grid (query blocks of 32, heads), four wavefronts each; the block with the most keys first.
// q, out: fp32 [n_queries][n_head][D]; query row t attends to keys [0, first_ctx + t).
// Keys are DK, values DV elements wide (one size D except where a latent's expanded keys carry a rotated part).
// kBias: the scores lose slope_h * distance, slope_h = 2^(-8 (h + 1) / n_head).  kRanged: a query sees a range of the keys, scores
// may be capped (then scale_log2e carries 2 log2 e scale / cap), the softmax may have a sink, the output may be gated.
// With either, the output is `dim` of DV elements per head in rows of ldo, fp32 or bf16.
enum { kCausal = 0, kBias = 1, kRanged = 2 };
struct PrefillExt {
    int dim = 0, ldo = 0, out_type = SKN_TYPE_F32;
    int tile0 = 0;  // the first tile of the operands
    skn_range range;
    int sink = 0;
    float cap_log2e = 0.f;
    const float* gate = nullptr;
    int ldg = 0;
};
template <int DK, int DV, int KIND>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK > 128 ? 1 : 2, DK > 128 ? 1 : 2))) void attn_prefill_kernel(const float* __restrict__ q, const u32x4* __restrict__ kfrag,
                                                          const u32x4* __restrict__ vfrag, float* __restrict__ out,
                                                          int n_queries, int n_head, int kv_group, int first_ctx, int n_tiles,
                                                          float scale_log2e, PrefillExt ext) {
    constexpr int KS = DK / 16, VS = DV / 16, DB = DV / 32;
    __shared__ float part[3][DB * 16 + 2][64];  // running maximum, sum and accumulators of wavefronts 1..3
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, h = lane >> 5, n = lane & 31;
    const int qb = (int)gridDim.x - 1 - (int)blockIdx.x, head = blockIdx.y;
    const int t = min(32 * qb + n, n_queries - 1);  // (rows past the end repeat the last one and are not stored)
    const int n_ctx = first_ctx + t;                // keys this lane's query sees
    // the last tile any query of the block needs
    const int tile0 = KIND == kRanged ? ext.tile0 : 0;
    const int last_tile = min((first_ctx + min(32 * qb + 31, n_queries - 1) - 1) >> 5, tile0 + n_tiles - 1);
    // the first tile its first query needs, and the first key this lane's query sees (a query's range starts no earlier than that
    // of the query before it)
    const int first_tile = KIND == kRanged ? ext.range.first(first_ctx + 32 * qb - 1) >> 5 : 0;
    const int first_key = KIND == kRanged ? ext.range.first(n_ctx - 1) : 0;

    // q as the column operand: lane 32 h + n holds elements 16 s + 8 h .. + 7 of query n, as an fp16 pair
    half8_t qh[KS], ql[KS];
    const float* qr = q + ((size_t)t * n_head + head) * DK + 8 * h;
#pragma unroll
    for (int s = 0; s < KS; s++) {
        const float4 a = *reinterpret_cast<const float4*>(qr + 16 * s), b = *reinterpret_cast<const float4*>(qr + 16 * s + 4);
        const float v[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
        for (int i = 0; i < 8; i++) {
            _Float16 x, y;
            skn_split_hilo(v[i] * scale_log2e, x, y);
            qh[s][i] = x, ql[s][i] = y;
        }
    }
    float16_t o[DB];
#pragma unroll
    for (int b = 0; b < DB; b++)
#pragma unroll
        for (int x = 0; x < 16; x++) o[b][x] = 0.f;
    const float slope = KIND == kBias ? exp2f(-8.0f * (float)(head + 1) / (float)n_head) * 1.4426950408889634f : 0.f;
    float mrun = -INFINITY, lrun = 0.f;  // running maximum (both halves agree) and this half's share of the sum

    // (grouped queries: kv_group consecutive query heads read the keys and values of one cached head)
    const u32x4* kp = kfrag + ((size_t)(head / kv_group) * n_tiles - tile0) * KS * 64 + lane;
    const u32x4* vp = vfrag + ((size_t)(head / kv_group) * n_tiles - tile0) * VS * 64 + lane;
    u32x4 kf[KS];
#pragma unroll
    for (int s = 0; s < KS; s++) kf[s] = kp[((size_t)min(first_tile + wave, last_tile) * KS + s) * 64];
    for (int tile = first_tile + wave; tile <= last_tile; tile += 4) {
        u32x4 vf[VS];
#pragma unroll
        for (int s = 0; s < VS; s++) vf[s] = vp[((size_t)tile * VS + s) * 64];
        // S^T = K Q^T: rows = keys of the tile, column = this lane's query (in units of log2 e)
        float16_t sc;
#pragma unroll
        for (int x = 0; x < 16; x++) sc[x] = 0.f;
#pragma unroll
        for (int s = 0; s < KS; s++) {
            const half8_t a = __builtin_bit_cast(half8_t, kf[s]);
            sc = __builtin_amdgcn_mfma_f32_32x32x16_f16(a, qh[s], sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_32x32x16_f16(a, ql[s], sc, 0, 0, 0);
        }
        // the next tile's keys (past the end: the last tile again, unused)
        const int nt = min(tile + 4, last_tile);
#pragma unroll
        for (int s = 0; s < KS; s++) kf[s] = kp[((size_t)nt * KS + s) * 64];
        // causal mask and the tile maximum of this query
        float mt = -INFINITY;
#pragma unroll
        for (int x = 0; x < 16; x++) {
            const int key = 32 * tile + 8 * (x >> 2) + 4 * h + (x & 3);
            if constexpr (KIND == kBias) sc[x] = fmaf(slope, (float)(key - (n_ctx - 1)), sc[x]);
            if constexpr (KIND == kRanged) {  // cap tanh(y) = cap (1 - 2 / (1 + exp(2 y)))
                if (ext.cap_log2e > 0.f) sc[x] = ext.cap_log2e * fmaf(-2.0f, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(sc[x])), 1.0f);
                sc[x] = key >= first_key ? sc[x] : -INFINITY;
            }
            sc[x] = key < n_ctx ? sc[x] : -INFINITY;
            mt = fmaxf(mt, sc[x]);
        }
        mt = fmaxf(mt, __shfl_xor(mt, 32));
        const float mnew = fmaxf(mrun, mt);
        // (a wavefront that has not met a visible key of this query yet: everything stays zero)
        const float alpha = mnew == -INFINITY ? 1.f : exp2f(mrun - mnew);
        mrun = mnew;
        float psum = 0.f;
        half8_t ph[2], pl[2];
#pragma unroll
        for (int x = 0; x < 16; x++) {
            const float p = mnew == -INFINITY ? 0.f : exp2f(sc[x] - mnew);
            psum += p;
            _Float16 a, b;
            skn_split_hilo(p, a, b);
            ph[x >> 3][x & 7] = a, pl[x >> 3][x & 7] = b;
        }
        lrun = lrun * alpha + psum;
        if (__any(alpha != 1.f)) {
#pragma unroll
            for (int b = 0; b < DB; b++)
#pragma unroll
                for (int x = 0; x < 16; x++) o[b][x] *= alpha;
        }
        // O^T += V^T P^T: rows = elements of the head, column = this lane's query
#pragma unroll
        for (int b = 0; b < DB; b++)
#pragma unroll
            for (int s = 0; s < 2; s++) {
                const half8_t a = __builtin_bit_cast(half8_t, vf[2 * b + s]);
                o[b] = __builtin_amdgcn_mfma_f32_32x32x16_f16(a, ph[s], o[b], 0, 0, 0);
                o[b] = __builtin_amdgcn_mfma_f32_32x32x16_f16(a, pl[s], o[b], 0, 0, 0);
            }
    }
    // merge: wavefronts 1..3 hand their state to wavefront 0 (every query sees itself: one of the four maxima is finite)
    if (wave > 0) {
        part[wave - 1][0][lane] = mrun;
        part[wave - 1][1][lane] = lrun;
#pragma unroll
        for (int b = 0; b < DB; b++)
#pragma unroll
            for (int x = 0; x < 16; x++) part[wave - 1][2 + 16 * b + x][lane] = o[b][x];
    }
    __syncthreads();
    if (wave > 0) return;
    {
        float mall = mrun;
#pragma unroll
        for (int w = 0; w < 3; w++) mall = fmaxf(mall, part[w][0][lane]);
        const float f0 = exp2f(mrun - mall);
        mrun = mall;
        lrun *= f0;
#pragma unroll
        for (int b = 0; b < DB; b++)
#pragma unroll
            for (int x = 0; x < 16; x++) o[b][x] *= f0;
#pragma unroll
        for (int w = 0; w < 3; w++) {
            const float mw = part[w][0][lane];
            const float f = mw == -INFINITY ? 0.f : exp2f(mw - mall);
            lrun += part[w][1][lane] * f;
#pragma unroll
            for (int b = 0; b < DB; b++)
#pragma unroll
                for (int x = 0; x < 16; x++) o[b][x] += part[w][2 + 16 * b + x][lane] * f;
        }
    }
    float ltot = lrun + __shfl_xor(lrun, 32);
    if (KIND == kRanged && ext.sink) ltot += exp2f(-mrun);
    const float inv = ltot > 0.f ? 1.0f / ltot : 0.f;
    if (KIND != kCausal && 32 * qb + n < n_queries) {
#pragma unroll
        for (int b = 0; b < DB; b++)
#pragma unroll
            for (int x = 0; x < 16; x++) {
                const int d = 32 * b + 8 * (x >> 2) + 4 * h + (x & 3);
                const size_t at = (size_t)t * ext.ldo + (size_t)head * ext.dim + d;
                if (d >= ext.dim) continue;
                float y = o[b][x] * inv;
                if (KIND == kRanged && ext.gate) y *= ext.gate[(size_t)t * ext.ldg + (size_t)head * ext.dim + d];
                if (ext.out_type == SKN_TYPE_F32) reinterpret_cast<float*>(out)[at] = y;
                else reinterpret_cast<uint16_t*>(out)[at] = skn_bf16_bits(y);
            }
    }
    if (KIND == kCausal && 32 * qb + n < n_queries) {
        float* orow = out + ((size_t)t * n_head + head) * DV + 4 * h;
#pragma unroll
        for (int b = 0; b < DB; b++)
#pragma unroll
            for (int g = 0; g < 4; g++)
                *reinterpret_cast<float4*>(orow + 32 * b + 8 * g) =
                    make_float4(o[b][4 * g] * inv, o[b][4 * g + 1] * inv, o[b][4 * g + 2] * inv, o[b][4 * g + 3] * inv);
    }
}

// workspace for the operands, grown on demand
int ensure_workspace(skn_ctx* ctx, size_t bytes) {
    if (bytes <= ctx->prefill_ws_bytes) return SKN_OK;
    SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    if (ctx->prefill_ws) SKN_HIP(ctx, hipFree(ctx->prefill_ws));
    ctx->prefill_ws = nullptr;
    ctx->prefill_ws_bytes = 0;
    hipError_t e = hipMalloc(&ctx->prefill_ws, bytes);
    if (e != hipSuccess) {
        (void)hipGetLastError();
        return skn_fail(ctx, SKN_ERR_OOM, "skn_attn_prefill: %zu bytes of workspace: %s", bytes, hipGetErrorString(e));
    }
    ctx->prefill_ws_bytes = bytes;
    return SKN_OK;
}

template <int D, int KIND>
int launch_prefill(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_dev, int n_queries, int first_ctx, float scale,
                   float* out_dev, int n_q_head, PrefillExt ext = PrefillExt()) {
    const int n_tokens = first_ctx + n_queries - 1;  // keys the last query sees
    const int n_tiles = (n_tokens + 31) / 32 - ext.tile0;
    const size_t frag_bytes = (size_t)kv->n_head * n_tiles * 32 * D * 2;
    SKN_TRY(ensure_workspace(ctx, 2 * frag_bytes));
    u32x4* kfrag = (u32x4*)ctx->prefill_ws;
    u32x4* vfrag = (u32x4*)((uint8_t*)ctx->prefill_ws + frag_bytes);
    skn_launch(ctx, attn_frag_kernel<D, KIND == kBias>, dim3(n_tiles, kv->n_head), dim3(256), 0, (const uint16_t*)kv->k_pool,
               (const uint16_t*)kv->v_pool, (const float*)kv->key_scale,
               (const int32_t*)(kv->page_table_dev + (size_t)seq * kv->pages_per_seq), kv->n_head,
               kv->page_tokens, n_tokens, ext.tile0, n_tiles, kfrag, vfrag);
    SKN_LAUNCH_CHECK(ctx);
    skn_launch(ctx, attn_prefill_kernel<D, D, KIND>, dim3((n_queries + 31) / 32, n_q_head), dim3(256), 0, q_dev, (const u32x4*)kfrag,
               (const u32x4*)vfrag, out_dev, n_queries, n_q_head, n_q_head / kv->n_head, first_ctx, n_tiles,
               scale * 1.4426950408889634f, ext);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

// attn_frag_kernel for keys and values that lie row by row (fp16): k [tokens][ldk], dim elements per head, beside rot [tokens][rot_dim]
// for all heads; v [tokens][ldv], vdim per head
template <int DK, int DV>
__global__ __launch_bounds__(256) void attn_frag_rows_kernel(const uint16_t* __restrict__ k, int ldk, const uint16_t* __restrict__ rot,
                                                             const uint16_t* __restrict__ v, int ldv, int dim, int rot_dim, int vdim, int n_tokens,
                                                             int n_tiles, u32x4* __restrict__ kfrag, u32x4* __restrict__ vfrag) {
    constexpr int kPitch = DV + 8;
    __shared__ __align__(16) uint16_t vt[32 * kPitch];
    const int tile = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    u32x4* kout = kfrag + ((size_t)head * n_tiles + tile) * (DK / 16) * 64;
    u32x4* vout = vfrag + ((size_t)head * n_tiles + tile) * (DV / 16) * 64;
    for (int i = tid; i < 32 * (DK / 8); i += 256) {
        const int r = i / (DK / 8), pc = i - r * (DK / 8), t = 32 * tile + r;
        uint32_t w[4] = {0u, 0u, 0u, 0u};
        if (t < n_tokens) {
            const uint16_t* kr = k + (size_t)t * ldk + (size_t)head * dim;
            const uint16_t* rr = rot + (size_t)t * rot_dim - dim;
            auto at = [&](int e) { return (uint32_t)(e < dim ? kr[e] : e < dim + rot_dim ? rr[e] : 0); };
            if (8 * pc + 8 <= dim && (dim & 7) == 0) {
                const u32x4 x = *reinterpret_cast<const u32x4*>(kr + 8 * pc);
                w[0] = x[0], w[1] = x[1], w[2] = x[2], w[3] = x[3];
            } else {
#pragma unroll
                for (int j = 0; j < 4; j++) w[j] = at(8 * pc + 2 * j) | (at(8 * pc + 2 * j + 1) << 16);
            }
        }
        kout[(pc >> 1) * 64 + 32 * (pc & 1) + r] = u32x4{w[0], w[1], w[2], w[3]};
    }
    for (int i = tid; i < 32 * DV; i += 256) {
        const int r = i / DV, d = i - r * DV, t = 32 * tile + r;
        vt[r * kPitch + d] = t < n_tokens && d < vdim ? v[(size_t)t * ldv + (size_t)head * vdim + d] : 0;
    }
    __syncthreads();
    for (int i = tid; i < (DV / 32) * 2 * 64; i += 256) {
        const int lane = i & 63, s = (i >> 6) & 1, b = i >> 7;
        const int h = lane >> 5, r = lane & 31;
        uint32_t w[4];
#pragma unroll
        for (int p = 0; p < 8; p += 2) {
            const uint32_t lo = vt[key_of(s, h, p) * kPitch + 32 * b + r], hi = vt[key_of(s, h, p + 1) * kPitch + 32 * b + r];
            w[p >> 1] = lo | (hi << 16);
        }
        vout[i] = u32x4{w[0], w[1], w[2], w[3]};
    }
}

PrefillExt ranged_ext(const skn_prefill_ranged& p, int tile0, float* scale) {
    PrefillExt ext;
    ext.dim = p.vdim;
    ext.ldo = p.ldo;
    ext.out_type = p.out_type;
    ext.tile0 = tile0;
    ext.range = p.range;
    ext.sink = p.sink;
    ext.gate = p.gate;
    ext.ldg = p.ldg;
    *scale = p.scale;
    if (p.softcap > 0.f) {
        ext.cap_log2e = p.softcap * 1.4426950408889634f;
        *scale = 2.0f * p.scale / p.softcap;
    }
    return ext;
}

template <int DK, int DV>
int launch_latent(skn_ctx* ctx, const uint16_t* k, int ldk, const uint16_t* rot, const uint16_t* v, int ldv, int dim, int rot_dim, int token0,
                  const float* q_prep, int n_queries, int pos0, int n_head, const skn_prefill_ranged& p) {
    const int n_tokens = pos0 + n_queries - token0, n_tiles = (n_tokens + 31) / 32;
    const size_t kbytes = (size_t)n_head * n_tiles * 32 * DK * 2, vbytes = (size_t)n_head * n_tiles * 32 * DV * 2;
    SKN_TRY(ensure_workspace(ctx, kbytes + vbytes));
    u32x4* kfrag = (u32x4*)ctx->prefill_ws;
    u32x4* vfrag = (u32x4*)((uint8_t*)ctx->prefill_ws + kbytes);
    skn_launch(ctx, attn_frag_rows_kernel<DK, DV>, dim3(n_tiles, n_head), dim3(256), 0, k, ldk, rot, v, ldv, dim, rot_dim, p.vdim, n_tokens, n_tiles, kfrag, vfrag);
    SKN_LAUNCH_CHECK(ctx);
    float scale;
    const PrefillExt ext = ranged_ext(p, token0 / 32, &scale);
    skn_launch(ctx, attn_prefill_kernel<DK, DV, kRanged>, dim3((n_queries + 31) / 32, n_head), dim3(256), 0, q_prep, (const u32x4*)kfrag, (const u32x4*)vfrag,
               (float*)p.out, n_queries, n_head, 1, pos0 + 1, n_tiles, scale * 1.4426950408889634f, ext);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

}  // namespace

bool skn_ranged_prefill_fits(const skn_kv* kv) { return kv->elem_type == SKN_TYPE_F16 && kv->head_dim <= 128; }

int skn_ranged_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_prep, int n_queries, int pos0, int n_head, const skn_prefill_ranged& p) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_RANGED && skn_ranged_prefill_fits(kv) && n_head % kv->n_head == 0, SKN_ERR_STATE,
                "prompt attention: not a ranged fp16 cache of heads up to 128");
    float scale;
    const PrefillExt ext = ranged_ext(p, p.range.first(pos0) >> 5, &scale);
    if (kv->head_dim == 64) return launch_prefill<64, kRanged>(ctx, kv, seq, q_prep, n_queries, pos0 + 1, scale, (float*)p.out, n_head, ext);
    return launch_prefill<128, kRanged>(ctx, kv, seq, q_prep, n_queries, pos0 + 1, scale, (float*)p.out, n_head, ext);
}

int skn_latent_prefill_width(int dim, int rot_dim, int vdim) {
    const int k = dim + rot_dim;
    if (rot_dim > 256) return 0;
    return k <= 64 && vdim <= 64 ? 64 : k <= 128 && vdim <= 128 ? 128 : k <= 192 && vdim <= 128 ? 192 : 0;
}

int skn_latent_prefill_launch(skn_ctx* ctx, const uint16_t* k, int ldk, const uint16_t* rot, const uint16_t* v, int ldv, int dim, int rot_dim, int token0,
                              const float* q_prep, int n_queries, int pos0, int n_head, const skn_prefill_ranged& p) {
    SKN_REQUIRE(ctx, token0 % 32 == 0 && token0 <= p.range.first(pos0), SKN_ERR_ARG, "prompt attention: keys from token %d on", token0);
    switch (skn_latent_prefill_width(dim, rot_dim, p.vdim)) {
        case 64: return launch_latent<64, 64>(ctx, k, ldk, rot, v, ldv, dim, rot_dim, token0, q_prep, n_queries, pos0, n_head, p);
        case 128: return launch_latent<128, 128>(ctx, k, ldk, rot, v, ldv, dim, rot_dim, token0, q_prep, n_queries, pos0, n_head, p);
        case 192: return launch_latent<192, 128>(ctx, k, ldk, rot, v, ldv, dim, rot_dim, token0, q_prep, n_queries, pos0, n_head, p);
        default: return skn_fail(ctx, SKN_ERR_SHAPE, "prompt attention: keys of %d + %d and values of %d elements", dim, rot_dim, p.vdim);
    }
}

// Shared with the decoder.  Query row t of n_queries attends to the first first_ctx + t tokens of sequence seq
// (first_ctx >= 1; all of them must be cached).  head_dim 64 or 128.
int skn_attn_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_dev, int n_queries, int first_ctx, float scale,
                            float* out_dev, int n_q_head) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_PLAIN, SKN_ERR_STATE, "attention: not a cache of fp16 keys and values (skn_attn_shared, _ranged and _latent read the others)");
    if (n_q_head <= 0) n_q_head = kv->n_head;
    SKN_REQUIRE(ctx, n_q_head % kv->n_head == 0, SKN_ERR_SHAPE,
                "attention: %d query heads are not a multiple of the %d cached heads", n_q_head, kv->n_head);
    if (kv->head_dim == 64) return launch_prefill<64, kCausal>(ctx, kv, seq, q_dev, n_queries, first_ctx, scale, out_dev, n_q_head);
    if (kv->head_dim == 128) return launch_prefill<128, kCausal>(ctx, kv, seq, q_dev, n_queries, first_ctx, scale, out_dev, n_q_head);
    return skn_fail(ctx, SKN_ERR_SHAPE, "skn_attn_prefill: head_dim %d is not supported (64 or 128)", kv->head_dim);
}

int skn_shared_attn_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_prep, int n_queries, int first_ctx, int n_head, float scale,
                                   void* out, int ldo, int out_type) {
    SKN_REQUIRE(ctx, kv->kind == SKN_KV_SHARED && kv->elem_type == SKN_TYPE_F16 && n_head % kv->n_head == 0, SKN_ERR_STATE, "prompt attention: not a shared fp16 cache");
    PrefillExt ext;
    ext.dim = kv->dim;
    ext.ldo = ldo;
    ext.out_type = out_type;
    if (kv->head_dim == 64) return launch_prefill<64, kBias>(ctx, kv, seq, q_prep, n_queries, first_ctx, scale, (float*)out, n_head, ext);
    if (kv->head_dim == 128) return launch_prefill<128, kBias>(ctx, kv, seq, q_prep, n_queries, first_ctx, scale, (float*)out, n_head, ext);
    return skn_fail(ctx, SKN_ERR_SHAPE, "prompt attention: head_dim %d is not supported (64 or 128)", kv->head_dim);
}

extern "C" int skn_attn_prefill(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_dev, int n_queries, float scale,
                                float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_attn_prefill: ctx is null");
    SKN_REQUIRE(ctx, kv != nullptr, SKN_ERR_ARG, "skn_attn_prefill: kv is null");
    SKN_REQUIRE(ctx, seq >= 0 && seq < kv->n_seq, SKN_ERR_RANGE, "skn_attn_prefill: sequence %d of %d", seq, kv->n_seq);
    SKN_REQUIRE(ctx, n_queries >= 0 && n_queries <= kv->len[seq], SKN_ERR_RANGE,
                "skn_attn_prefill: %d query rows for a sequence holding %d tokens", n_queries, kv->len[seq]);
    if (n_queries == 0) return SKN_OK;
    SKN_REQUIRE(ctx, q_dev && out_dev, SKN_ERR_ARG, "skn_attn_prefill: null pointer");
    SKN_REQUIRE(ctx, ((uintptr_t)q_dev & 15) == 0 && ((uintptr_t)out_dev & 15) == 0, SKN_ERR_ARG,
                "skn_attn_prefill: q and out must be 16-byte aligned");
    return skn_attn_prefill_launch(ctx, kv, seq, q_dev, n_queries, kv->len[seq] - n_queries + 1, scale, out_dev);
}
